// Causal softmax attention over the paged cache with a bias by distance and a query temperature,
// keys and values of different sizes, for gfx950.
//
//     score(i, j) = (q_i . k_j) * scale * temp(i) + bias[i - j, head]      for j <= i
//     temp(p) = 1 + coef * ln(floor((p + 1) / every) + 1)
//
// `bias` is a float32 table [distances, heads] that the host has laid out from the learned rows (one
// row for every distance up to the model's last position), so the kernel needs no logarithm a score.
// Pools are [page, kv_head, slot_in_page, size] with size dk for keys and dv for values.
//
// A window (`window` > 0) narrows what a query sees to its last `window` keys, its own among them, plus the
// first `keep_first` keys of its sequence, which stay visible for good: j <= i and (i - j < window or j < keep_first).
// The kernels then walk only the tiles of 64 keys that hold such keys: the tiles of the kept first keys, then the
// tiles from the one in which the window of the tile's first token starts (`KeyWalk`).  `out_scale` multiplies the
// normalised output (a mixer that is one of several side by side has a weight of its own).
//
// Chunks (`chunk` > 0) narrow it otherwise: i sees j <= i only where floor(i / chunk) = floor(j / chunk), chunks being
// counted from a sequence's position 0.  `softcap` c > 0 bends a scaled score s to c tanh(s / c).
//
// Maps (`maps` m > 1): every kv head holds m keys a slot, side by side in its row [m * dk], and one value; the query
// heads come in the order [kv head][map][head of the group], and an attention of its own runs for every (kv head, map)
// over that map's keys and the kv head's values: H counts the query heads of all maps, G the (kv head, map) pairs.  What
// becomes of the maps' outputs is up to `merge_maps`, which takes them as the kernels leave unfinished rows.
//
// A gate (`Gate`): an output channel c of head h is multiplied by sigmoid(g[token, (h * dv + c) / every]) when its row is
// finished, the pre-activations g float32 rows (some columns of the projections the queries came from).
//
// A sink (`sink`, float32 [heads], or null) is one more term exp(sink[head]) in a row's denominator, with no key and
// no value: the weights of a row then sum to less than one.  It counts once a row, whatever the number of runs: the
// kernels add it when a row is finished (a row in runs: when the runs are merged).
//
// One workgroup of four wavefronts takes a tile of consecutive tokens of one sequence and (a chunk of)
// the query heads of one kv head: 16 rows of (token, head), four a wavefront.  64 keys and values at a
// time are staged in LDS as float32 for the whole workgroup; a lane owns one key of the 64 for the
// scores of its wavefront's four rows, then one value channel (and the ones 64 further on) for the
// weighted sum.  Everything is float32; the softmax is the running one (maximum, sum, rescaled sum).
#include "common.h"

#include <algorithm>
#include <cmath>
#include <type_traits>

#define ROWS_PER_WAVE 4
#define WAVES 4
#define ROWS (ROWS_PER_WAVE * WAVES)
#define KEYS 64
#define MAX_VCHUNKS 4          // value channels a lane owns at most: dv <= 256

// Which tiles of KEYS keys a tile of queries (positions first_pos .. last_pos) walks: step v < kept is tile v (the kept
// first keys), step v >= kept the tile at `start + (v - kept) * KEYS`.  Without a window: every tile from key 0.
struct KeyWalk {
    int kept, start, steps;
    __device__ __forceinline__ KeyWalk(int first_pos, int last_pos, int window, int keep_first, int chunk) {
        kept = 0;
        start = chunk > 0 ? first_pos / chunk * chunk / KEYS * KEYS : 0;
        if (window > 0) {
            const int lo = max(first_pos - window + 1, 0) / KEYS * KEYS;       // the tile in which the first row's window starts
            const int kept_end = (min(keep_first, last_pos + 1) + KEYS - 1) / KEYS * KEYS;
            if (lo > kept_end) { kept = kept_end / KEYS; start = lo; }
        }
        steps = kept + (last_pos - start) / KEYS + 1;
    }
    __device__ __forceinline__ int first_key(int v) const { return v < kept ? v * KEYS : start + (v - kept) * KEYS; }
};

// the first key of the run of neighbouring keys that a query at `pos` sees (the kept first keys come besides)
__device__ __forceinline__ int first_seen(int pos, int window, int chunk) {
    return chunk > 0 ? pos / chunk * chunk : window > 0 ? pos - window + 1 : 0;
}

__device__ __forceinline__ bool key_seen(int key, int pos, int lo, int keep_first) {
    return key <= pos && (key >= lo || key < keep_first);
}

// cap * tanh(s / cap): near zero tanh's own series (its next term is below 1e-8 of the value at 1/4), elsewhere
// 1 - 2 / (e^2x + 1), which tends to 1 where the exponential overflows
__device__ __forceinline__ float soft_capped(float s, float cap, float inv_cap) {
    const float x = fabsf(s) * inv_cap, x2 = x * x;
    const float near = x * (1.0f + x2 * (-1.0f / 3.0f + x2 * (2.0f / 15.0f + x2 * (-17.0f / 315.0f + x2 * (62.0f / 2835.0f)))));
    const float far = 1.0f - 2.0f / (expf(2.0f * x) + 1.0f);
    return copysignf(cap * (x < 0.25f ? near : far), s);
}

// keys and values of the step's tokens into their places in the pages
template <typename T>
__global__ void kv_store_kernel(const T* __restrict__ qkv, int row_stride, int k_off, int v_off,
                                const int32_t* __restrict__ slot_mapping, T* __restrict__ kpool, T* __restrict__ vpool,
                                int G, int dk, int dv, int page_size) {
    const int t = blockIdx.x;
    const int slot = slot_mapping[t];
    if (slot < 0) return;
    const int page = slot / page_size, in_page = slot % page_size;
    const T* row = qkv + static_cast<size_t>(t) * row_stride;
    for (int i = threadIdx.x; i < G * dk; i += blockDim.x) {
        const int g = i / dk, c = i % dk;
        kpool[((static_cast<size_t>(page) * G + g) * page_size + in_page) * dk + c] = row[k_off + i];
    }
    for (int i = threadIdx.x; i < G * dv; i += blockDim.x) {
        const int g = i / dv, c = i % dv;
        vpool[((static_cast<size_t>(page) * G + g) * page_size + in_page) * dv + c] = row[v_off + i];
    }
}

// The same for projections that still want their norm and rotation, all of it in float32:
//   q <- rotate(rmsnorm(q) * wq), k <- rotate(rmsnorm(k) * wk)
//   The norms (a null weight: no norm) run over the WHOLE projection of a token, all heads at once, weights [H * dq]
//   and [G * dk]; or, `per_head`, over every head on its own with one weight [dq] (or [k_normed]) shared by the heads.
//   Of a key head only the first `k_normed` channels are normed (whole-projection norms: all of them); the others
//   pass as projected.
//   The rotation (a null freq: none) turns `rot` channels of every head, from channel `rot_at_q` (queries) or
//   `rot_at_k` (keys) on, by the angles position * freq[p], cos and sin times `amplitude`: channel c of them with
//   channel c + rot/2, or, `adjacent`, channel 2p with channel 2p + 1.  The other channels pass as they are.
// proj float32 [T, row_stride] holds q [H * dq] | k [G * dk] | v [G * dv] (`v_from_k`: no v; the values are the keys as
// projected, before their norm, and dv = dk); q goes to q_out [T, H * dq] in the compute
// type, k and v into their page slots.  A token is taken by gridDim.y workgroups, each with its share of the elements
// (and the sums of squares, which every one of them works out): one for steps of many
// tokens; a step of few tokens, where one workgroup a token would walk its row alone, spreads the row.
#define ROT_PAIRS 128          // rotated pairs of a head at most: heads of up to 256 rotated channels
#define NORM_HEADS 1024        // heads of queries and keys together that are normed one by one, at most

struct QkForm {
    int H, G, dq, dk, dv, k_normed, rot, rot_at_q, rot_at_k;
    bool v_from_k, per_head, adjacent;
};

template <typename T>
__global__ void __launch_bounds__(256)
qk_norm_rope_store_kernel(const float* __restrict__ proj, int row_stride, const int32_t* __restrict__ positions,
                          const int32_t* __restrict__ slot_mapping, const float* __restrict__ wq, const float* __restrict__ wk,
                          float eps, const float* __restrict__ freq, float amplitude, T* __restrict__ q_out,
                          T* __restrict__ kpool, T* __restrict__ vpool, int page_size, QkForm f) {
    __shared__ float scratch[8];
    __shared__ float cos_of[ROT_PAIRS], sin_of[ROT_PAIRS];     // the token's angles, worked out once for all heads
    __shared__ float head_r[NORM_HEADS];                       // per_head: 1 / rms of every query head, then of every key head
    const int t = blockIdx.x, tid = threadIdx.x;
    const float* row = proj + static_cast<size_t>(t) * row_stride;
    const int H = f.H, G = f.G, dq = f.dq, dk = f.dk, dv = f.dv, rot = f.rot;
    const int nq = H * dq, nk = G * dk;
    const int slices = gridDim.y, slice = blockIdx.y;
    const int per = ((nq + nk + slices - 1) / slices + 3) / 4 * 4;
    float rq = 1.f, rk = 1.f;
    if (f.per_head) {
        // a head a wavefront at a time: its lanes walk the head's normed channels; only heads of this workgroup's share
        const int lane = tid & (WAVE - 1), wave = tid / WAVE, waves = blockDim.x / WAVE;
        auto head_of = [&](int i) { return i < nq ? i / dq : H + (i - nq) / dk; };
        const int i0 = slice * per, i1 = min(nq + nk, (slice + 1) * per);
        for (int hd = i0 < i1 ? head_of(i0) + wave : H + G; hd <= (i0 < i1 ? head_of(i1 - 1) : -1); hd += waves) {
            const bool is_q = hd < H;
            const float* w = is_q ? wq : wk;
            if (!w) continue;                                  // the same for the whole wavefront
            const float* src = is_q ? row + hd * dq : row + nq + (hd - H) * dk;
            const int n = is_q ? dq : f.k_normed;
            float ss = 0.f;
            for (int c = lane; c < n; c += WAVE) ss += src[c] * src[c];
            ss = wave_sum(ss);
            if (lane == 0) head_r[hd] = 1.0f / sqrtf(ss / static_cast<float>(n) + eps);
        }
        __syncthreads();
    } else {
        if (wq) {
            float ss = 0.f;
            for (int i = tid; i < nq; i += blockDim.x) ss += row[i] * row[i];
            rq = 1.0f / sqrtf(block_sum(ss, scratch) / static_cast<float>(nq) + eps);
        }
        if (wk) {
            float ss = 0.f;
            for (int i = tid; i < nk; i += blockDim.x) ss += row[nq + i] * row[nq + i];
            rk = 1.0f / sqrtf(block_sum(ss, scratch) / static_cast<float>(nk) + eps);
        }
    }
    const float pos = static_cast<float>(positions[t]);
    const int half = rot / 2;
    if (freq) {
        for (int p = tid; p < half; p += blockDim.x) {
            float sn, cs;
            sincosf(pos * freq[p], &sn, &cs);
            cos_of[p] = cs * amplitude;
            sin_of[p] = sn * amplitude;
        }
        __syncthreads();
    }
    const int slot = slot_mapping ? slot_mapping[t] : -1;
    const int page = slot >= 0 ? slot / page_size : 0, in_page = slot >= 0 ? slot % page_size : 0;
    for (int i = slice * per + tid; i < min(nq + nk, (slice + 1) * per); i += blockDim.x) {
        const bool is_q = i < nq;
        const int j = is_q ? i : i - nq;                 // index inside the projection
        const float* src = is_q ? row : row + nq;
        const float* w = is_q ? wq : wk;
        const int size = is_q ? dq : dk;
        const int hd = j / size, c = j - hd * size;
        const int normed = !w ? 0 : (is_q ? size : f.k_normed);       // leading channels of the head that are normed
        const float r = f.per_head ? (w ? head_r[is_q ? hd : H + hd] : 1.f) : (is_q ? rq : rk);
        // the element at channel cc of this head, after its norm
        auto normed_at = [&](int cc) -> float {
            const float x = src[hd * size + cc];
            return cc < normed ? x * r * w[f.per_head ? cc : hd * size + cc] : x;
        };
        float v = normed_at(c);
        const int cr = c - (is_q ? f.rot_at_q : f.rot_at_k);           // index among the rotated channels
        if (freq && cr >= 0 && cr < rot) {
            const bool first = f.adjacent ? !(cr & 1) : cr < half;
            const int partner = f.adjacent ? (cr ^ 1) : (first ? cr + half : cr - half);
            const int p = f.adjacent ? (cr >> 1) : (first ? cr : cr - half);
            const float other = normed_at(c - cr + partner);
            const float cs = cos_of[p], sn = sin_of[p];
            v = first ? v * cs - other * sn : v * cs + other * sn;
        }
        if (is_q) {
            st(q_out + static_cast<size_t>(t) * nq + j, v);
        } else if (slot >= 0) {
            st(kpool + ((static_cast<size_t>(page) * G + hd) * page_size + in_page) * dk + c, v);
        }
    }
    if (slot >= 0) {
        const float* vsrc = f.v_from_k ? row + nq : row + nq + nk;      // the values may be the keys as projected, before their norm
        const int vper = (G * dv + slices - 1) / slices;
        for (int i = slice * vper + tid; i < min(G * dv, (slice + 1) * vper); i += blockDim.x) {
            const int g = i / dv, c = i % dv;
            st(vpool + ((static_cast<size_t>(page) * G + g) * page_size + in_page) * dv + c, vsrc[i]);
        }
    }
}

// The same with norms a head (or none), for heads of up to 64 SL channels: a wavefront takes HB heads at once, whose channels
// lie in its lanes (channel lane + 64 u in slot u), so a head is read once, normed, rotated through the wavefront's own LDS
// and stored; what the HB heads wait for they wait for together.
template <typename T, int SL, int HB>
__global__ void __launch_bounds__(256)
qk_heads_kernel(const float* __restrict__ proj, int row_stride, const int32_t* __restrict__ positions,
                const int32_t* __restrict__ slot_mapping, const float* __restrict__ wq, const float* __restrict__ wk,
                float eps, const float* __restrict__ freq, float amplitude, T* __restrict__ q_out,
                T* __restrict__ kpool, T* __restrict__ vpool, int page_size, QkForm f) {
    __shared__ float cos_of[ROT_PAIRS], sin_of[ROT_PAIRS];
    __shared__ float turned[4][HB][64 * SL];
    const int t = blockIdx.x, tid = threadIdx.x, lane = tid & (WAVE - 1), wave = tid / WAVE;
    const float* row = proj + static_cast<size_t>(t) * row_stride;
    const int H = f.H, G = f.G, dq = f.dq, dk = f.dk, dv = f.dv, half = f.rot / 2;
    const int slices = gridDim.y, slice = blockIdx.y;
    if (freq) {
        const float pos = static_cast<float>(positions[t]);
        for (int p = tid; p < half; p += blockDim.x) {
            float sn, cs;
            sincosf(pos * freq[p], &sn, &cs);
            cos_of[p] = cs * amplitude;
            sin_of[p] = sn * amplitude;
        }
        __syncthreads();
    }
    const int slot = slot_mapping ? slot_mapping[t] : -1;
    const int page = slot >= 0 ? slot / page_size : 0, in_page = slot >= 0 ? slot % page_size : 0;
    float weight_q[SL], weight_k[SL];
#pragma unroll
    for (int u = 0; u < SL; ++u) {
        const int c = lane + 64 * u;
        weight_q[u] = wq && c < dq ? wq[c] : 0.f;
        weight_k[u] = wk && c < f.k_normed ? wk[c] : 0.f;
    }
    const int per = (H + G + slices - 1) / slices, first = slice * per, last = min(H + G, first + per);
    for (int base = first + wave * HB; base < last; base += 4 * HB) {
        float x[HB][SL], ss[HB];
#pragma unroll
        for (int b = 0; b < HB; ++b) {
            const int hd = min(base + b, last - 1);              // (a head too many is read again and not stored)
            const bool is_q = hd < H;
            const float* src = is_q ? row + hd * dq : row + H * dq + (hd - H) * dk;
            const int n = is_q ? dq : dk;
#pragma unroll
            for (int u = 0; u < SL; ++u) x[b][u] = lane + 64 * u < n ? src[lane + 64 * u] : 0.f;
        }
#pragma unroll
        for (int b = 0; b < HB; ++b) {
            const int normed = min(base + b, last - 1) < H ? dq : f.k_normed;
            ss[b] = 0.f;
#pragma unroll
            for (int u = 0; u < SL; ++u) ss[b] += lane + 64 * u < normed ? x[b][u] * x[b][u] : 0.f;
        }
#pragma unroll
        for (int b = 0; b < HB; ++b) ss[b] = wave_sum(ss[b]);
#pragma unroll
        for (int b = 0; b < HB; ++b) {
            const bool is_q = min(base + b, last - 1) < H;
            const int normed = !(is_q ? wq : wk) ? 0 : is_q ? dq : f.k_normed;
            const float r = normed > 0 ? 1.0f / sqrtf(ss[b] / static_cast<float>(normed) + eps) : 1.f;
#pragma unroll
            for (int u = 0; u < SL; ++u)
                if (lane + 64 * u < normed) x[b][u] = x[b][u] * r * (is_q ? weight_q[u] : weight_k[u]);
        }
        if (freq) {
            __builtin_amdgcn_wave_barrier();      // a wavefront reads only what it wrote itself, and its LDS accesses stay in order
#pragma unroll
            for (int b = 0; b < HB; ++b)
#pragma unroll
                for (int u = 0; u < SL; ++u) turned[wave][b][lane + 64 * u] = x[b][u];
            __builtin_amdgcn_wave_barrier();
#pragma unroll
            for (int b = 0; b < HB; ++b) {
                const int at = min(base + b, last - 1) < H ? f.rot_at_q : f.rot_at_k;
#pragma unroll
                for (int u = 0; u < SL; ++u) {
                    const int cr = lane + 64 * u - at;
                    if (cr >= 0 && cr < f.rot) {
                        const bool one = f.adjacent ? !(cr & 1) : cr < half;
                        const int partner = f.adjacent ? (cr ^ 1) : (one ? cr + half : cr - half);
                        const int p = f.adjacent ? (cr >> 1) : (one ? cr : cr - half);
                        const float other = turned[wave][b][at + partner], cs = cos_of[p], sn = sin_of[p];
                        x[b][u] = one ? x[b][u] * cs - other * sn : x[b][u] * cs + other * sn;
                    }
                }
            }
        }
#pragma unroll
        for (int b = 0; b < HB; ++b) {
            const int hd = base + b;
            if (hd >= last || (hd >= H && slot < 0)) continue;
            T* dst = hd < H ? q_out + (static_cast<size_t>(t) * H + hd) * dq
                            : kpool + ((static_cast<size_t>(page) * G + (hd - H)) * page_size + in_page) * dk;
            const int n = hd < H ? dq : dk;
#pragma unroll
            for (int u = 0; u < SL; ++u)
                if (lane + 64 * u < n) st(dst + lane + 64 * u, x[b][u]);
        }
    }
    if (slot >= 0) {
        const float* vsrc = row + H * dq + (f.v_from_k ? 0 : G * dk);      // the values may be the keys as projected
        const int vper = (G * dv + slices - 1) / slices;
        for (int i = slice * vper + tid; i < min(G * dv, (slice + 1) * vper); i += blockDim.x) {
            const int g = i / dv, c = i - g * dv;
            st(vpool + ((static_cast<size_t>(page) * G + g) * page_size + in_page) * dv + c, vsrc[i]);
        }
    }
}

template <typename T>
static void launch_qk_heads(const float* proj, int row_stride, const int32_t* positions, const int32_t* slot_mapping, const float* wq,
                            const float* wk, float eps, const float* freq, float amplitude, T* q_out, T* kpool, T* vpool, int page_size,
                            const QkForm& f, int Tn, hipStream_t stream) {
    const int size = std::max(f.H > 0 ? f.dq : 0, f.G > 0 ? f.dk : 0);
    // few tokens: one head a wavefront; many: every workgroup a row of its own, as long as that fills the chip
    const int slices = std::max(1, std::min({16, (f.H + f.G + 3) / 4, 2048 / std::max(Tn, 1)}));
    const dim3 grid(Tn, slices);
    if (size <= 64)
        qk_heads_kernel<T, 1, 4><<<grid, 256, 0, stream>>>(proj, row_stride, positions, slot_mapping, wq, wk, eps, freq, amplitude, q_out, kpool, vpool, page_size, f);
    else if (size <= 128)
        qk_heads_kernel<T, 2, 2><<<grid, 256, 0, stream>>>(proj, row_stride, positions, slot_mapping, wq, wk, eps, freq, amplitude, q_out, kpool, vpool, page_size, f);
    else
        qk_heads_kernel<T, 4, 2><<<grid, 256, 0, stream>>>(proj, row_stride, positions, slot_mapping, wq, wk, eps, freq, amplitude, q_out, kpool, vpool, page_size, f);
}

// `per_head`, `adjacent`, `dq`, `k_normed`, `rot_at_q`, `rot_at_k`: see the kernel.  G may be 0 (queries alone).
NI_EXPORT int ni_qk_norm_rope_store(const void* proj, int row_stride, const void* positions, const void* slot_mapping,
                                    const void* wq, const void* wk, float eps, const void* freq, int rot, float amplitude,
                                    void* q_out, void* kpool, void* vpool, int T, int H, int G, int dq, int dk, int dv, int page_size,
                                    int v_from_k, int per_head, int k_normed, int rot_at_q, int rot_at_k, int adjacent,
                                    int dtype, hipStream_t stream) {
    if (T <= 0) return 0;
    if (H < 0 || G < 0 || dq < 0 || dk < 0 || dv < 0 || (H > 0 && dq < 1) || (G > 0 && dk < 1)) return -1;
    if (rot < 0 || rot % 2 || rot > 2 * ROT_PAIRS || rot_at_q < 0 || rot_at_k < 0) return -1;
    if (freq && ((H > 0 && rot_at_q + rot > dq) || (G > 0 && rot_at_k + rot > dk))) return -1;
    if (row_stride < H * dq + G * dk + (v_from_k ? 0 : G * dv)) return -1;
    if (v_from_k && dv != dk) return -1;
    if (k_normed < 0 || k_normed > dk || (!per_head && wk && k_normed != dk)) return -1;
    if (per_head && H + G > NORM_HEADS) return -1;
    if ((H > 0 && !q_out) || (G > 0 && slot_mapping && (!kpool || (dv > 0 && !vpool)))) return -1;
    const QkForm f{H, G, dq, dk, dv, k_normed, freq ? rot : 0, rot_at_q, rot_at_k, v_from_k != 0, per_head != 0, adjacent != 0};
    if ((per_head || (!wq && !wk)) && std::max(H > 0 ? dq : 0, G > 0 ? dk : 0) <= 4 * WAVE) {
        if (dtype == 0)
            launch_qk_heads<float>((const float*)proj, row_stride, (const int32_t*)positions, (const int32_t*)slot_mapping, (const float*)wq,
                                   (const float*)wk, eps, (const float*)freq, amplitude, (float*)q_out, (float*)kpool, (float*)vpool, page_size, f, T, stream);
        else
            launch_qk_heads<bf16_t>((const float*)proj, row_stride, (const int32_t*)positions, (const int32_t*)slot_mapping, (const float*)wq,
                                    (const float*)wk, eps, (const float*)freq, amplitude, (bf16_t*)q_out, (bf16_t*)kpool, (bf16_t*)vpool, page_size, f, T,
                                    stream);
        return NI_LAUNCH_RESULT();
    }
    // few tokens: a row's elements over several workgroups, one pass of 256 threads each
    const int slices = T >= 64 ? 1 : std::max(1, std::min(16, (H * dq + G * dk + 255) / 256));
    const dim3 grid(T, slices);
    if (dtype == 0)
        qk_norm_rope_store_kernel<float><<<grid, 256, 0, stream>>>((const float*)proj, row_stride, (const int32_t*)positions,
            (const int32_t*)slot_mapping, (const float*)wq, (const float*)wk, eps, (const float*)freq, amplitude,
            (float*)q_out, (float*)kpool, (float*)vpool, page_size, f);
    else
        qk_norm_rope_store_kernel<bf16_t><<<grid, 256, 0, stream>>>((const float*)proj, row_stride, (const int32_t*)positions,
            (const int32_t*)slot_mapping, (const float*)wq, (const float*)wk, eps, (const float*)freq, amplitude,
            (bf16_t*)q_out, (bf16_t*)kpool, (bf16_t*)vpool, page_size, f);
    return NI_LAUNCH_RESULT();
}

// 64 rows of a pool (keys or values of one kv head) from their pages into LDS as float32, row stride `stride`: `size`
// channels of rows of `row` (the pool is handed over at the first of them).
// With `pieces` (rows of whole 16-byte pieces, 16-byte aligned) a thread asks for four pieces before it stores
// the first: the loads of a tile are then in flight together instead of one round trip after the other.
template <typename T>
__device__ __forceinline__ void stage_rows(const T* __restrict__ pool, float* __restrict__ dst, int stride, int size, int row,
                                           const int32_t* __restrict__ table, int page_size, int G, int g, int k0,
                                           int k_last, bool pieces) {
    constexpr int VEC = 16 / sizeof(T);
    const int tid = threadIdx.x, threads = blockDim.x;
    if (pieces) {
        const int per_row = size / VEC, total = KEYS * per_row;
        for (int base = 0; base < total; base += 4 * threads) {
            RawRow<T, VEC> raw[4];
            bool have[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const int idx = base + u * threads + tid;
                have[u] = false;
                if (idx < total) {
                    const int j = idx / per_row, pc = idx % per_row, key = k0 + j;
                    if (key <= k_last) {
                        const int page = table[key / page_size];
                        if (page >= 0) {
                            raw[u].load(pool + ((static_cast<size_t>(page) * G + g) * page_size + key % page_size) * row + pc * VEC);
                            have[u] = true;
                        }
                    }
                }
            }
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const int idx = base + u * threads + tid;
                if (idx < total) {
                    float* d = dst + (idx / per_row) * stride + (idx % per_row) * VEC;
#pragma unroll
                    for (int e = 0; e < VEC; ++e) d[e] = have[u] ? raw[u].get(e) : 0.f;
                }
            }
        }
        return;
    }
    for (int i = tid; i < KEYS * size; i += threads) {
        const int j = i / size, c = i % size, key = k0 + j;
        float v = 0.f;
        if (key <= k_last) {
            const int page = table[key / page_size];
            if (page >= 0) v = ld(pool + ((static_cast<size_t>(page) * G + g) * page_size + key % page_size) * row + c);
        }
        dst[j * stride + c] = v;
    }
}

// The same in two halves, for tiles whose rows are at most four 16-byte pieces a thread: what stage_rows would
// load, asked for and kept in registers, and its way into LDS afterwards.  Keys and values asked for one after the
// other and stored after both are on their way together: one round trip to memory a tile instead of two.
template <typename T> struct StagedRows {
    RawRow<T, 16 / sizeof(T)> raw[4];
    bool have[4];
};

template <typename T>
__device__ __forceinline__ void stage_ask(const T* __restrict__ pool, StagedRows<T>& x, int size, int row, const int32_t* __restrict__ table,
                                          int page_size, int G, int g, int k0, int k_last) {
    constexpr int VEC = 16 / sizeof(T);
    const int tid = threadIdx.x, threads = blockDim.x;
    const int per_row = size / VEC, total = KEYS * per_row;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
        const int idx = u * threads + tid;
        x.have[u] = false;
        if (idx < total) {
            const int j = idx / per_row, pc = idx % per_row, key = k0 + j;
            if (key <= k_last) {
                const int page = table[key / page_size];
                if (page >= 0) {
                    x.raw[u].load(pool + ((static_cast<size_t>(page) * G + g) * page_size + key % page_size) * row + pc * VEC);
                    x.have[u] = true;
                }
            }
        }
    }
}

template <typename T>
__device__ __forceinline__ void stage_put(const StagedRows<T>& x, float* __restrict__ dst, int stride, int size) {
    constexpr int VEC = 16 / sizeof(T);
    const int tid = threadIdx.x, threads = blockDim.x;
    const int per_row = size / VEC, total = KEYS * per_row;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
        const int idx = u * threads + tid;
        if (idx < total) {
            float* d = dst + (idx / per_row) * stride + (idx % per_row) * VEC;
#pragma unroll
            for (int e = 0; e < VEC; ++e) d[e] = x.have[u] ? x.raw[u].get(e) : 0.f;
        }
    }
}

// keys and values of a tile into LDS: together where both fit four pieces a thread, else one after the other
template <typename T>
__device__ __forceinline__ void stage_tile(const T* __restrict__ kpool, const T* __restrict__ vpool, float* __restrict__ Ks, int dkp,
                                           int dk, int k_row, float* __restrict__ Vs, int dvp, int dv, const int32_t* __restrict__ table,
                                           int page_size, int G, int g, int k0, int k_last, bool k_pieces, bool v_pieces) {
    constexpr int VEC = 16 / sizeof(T);
    const int room = 4 * blockDim.x;
    if (k_pieces && v_pieces && KEYS * (dk / VEC) <= room && KEYS * (dv / VEC) <= room) {
        StagedRows<T> k, v;
        stage_ask<T>(kpool, k, dk, k_row, table, page_size, G, g, k0, k_last);
        stage_ask<T>(vpool, v, dv, dv, table, page_size, G, g, k0, k_last);
        stage_put<T>(k, Ks, dkp, dk);
        stage_put<T>(v, Vs, dvp, dv);
        return;
    }
    stage_rows<T>(kpool, Ks, dkp, dk, k_row, table, page_size, G, g, k0, k_last, k_pieces);
    stage_rows<T>(vpool, Vs, dvp, dv, dv, table, page_size, G, g, k0, k_last, v_pieces);
}

// The gate on an attention's output: see the top of the file (null rows: none)
struct Gate {
    const float* rows;
    int stride, every;
    // the factor on channel c of the H * dv of token t
    __device__ __forceinline__ float of(size_t t, int c) const {
        return rows ? 1.0f / (1.0f + expf(-rows[t * stride + (every == 1 ? c : c / every)])) : 1.f;
    }
};

// What an attention may do beside the bias: see the top of the file (0, 0, 1: nothing)
struct ScoreForm {
    float softcap;
    int chunk, maps;
};

template <typename T>
__global__ void __launch_bounds__(WAVES * WAVE)
bias_attention_kernel(const T* __restrict__ qkv, int row_stride, const T* __restrict__ kpool, const T* __restrict__ vpool,
                      const int32_t* __restrict__ block_table, int table_width, const int32_t* __restrict__ tiles,
                      const int32_t* __restrict__ positions, const float* __restrict__ bias, int distances, T* __restrict__ out, int H, int G, int dk, int dv,
                      int page_size, float scale, float temp_coef, int temp_every, int heads_per_chunk, int n_runs,
                      float* __restrict__ partial, bool k_pieces, bool v_pieces, int dkp, int window, int keep_first,
                      float out_scale, const float* __restrict__ sink, ScoreForm form, Gate gate) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    // a lane reads its key's row: the stride is the row plus four floats where rows are whole 16-byte pieces (read
    // as such), plus one otherwise; both spread the lanes over the banks
    float* Qs = lds;                              // [ROWS][dk]
    float* Ks = Qs + ROWS * dk;                   // [KEYS][dkp]
    float* Vs = Ks + KEYS * dkp;                  // [KEYS][dv]
    float* Ps = Vs + KEYS * dv;                   // [WAVES][ROWS_PER_WAVE][KEYS]
    // with n_runs > 1 the keys of a tile are cut into runs, one workgroup each, whose (maximum, sum, weighted
    // sum) a second kernel merges: a single token over thousands of keys then fills the chip
    const int tile = blockIdx.x / n_runs, run = blockIdx.x % n_runs, g = blockIdx.y, chunk = blockIdx.z;
    // the first position is read from the step's positions, not from the tile: a recorded decode step is replayed
    // with new positions and the tiles it was recorded with
    const int seq = tiles[4 * tile], first_row = tiles[4 * tile + 1], n_tok = tiles[4 * tile + 2];
    const int first_pos = positions[first_row];
    const int group = H / G;
    const int heads_here = std::min(heads_per_chunk, group - chunk * heads_per_chunk);
    const int head0 = g * group + chunk * heads_per_chunk;
    const int n_rows = n_tok * heads_here;        // row r = token r / heads_here, head r % heads_here
    const int tid = threadIdx.x, lane = tid & (WAVE - 1), wave = tid / WAVE;
    // the kv head whose pages hold this head's keys and values, and where its map's keys lie in a row of keys
    const int kv = g / form.maps, kv_heads = G / form.maps, k_row = form.maps * dk;
    kpool += (g % form.maps) * dk;
    const float inv_cap = form.softcap > 0.f ? 1.0f / form.softcap : 0.f;

    for (int i = tid; i < ROWS * dk; i += blockDim.x) {
        const int r = i / dk, c = i % dk;
        float v = 0.f;
        if (r < n_rows)
            v = ld(qkv + static_cast<size_t>(first_row + r / heads_here) * row_stride + (head0 + r % heads_here) * dk + c);
        Qs[i] = v;
    }
    float m[ROWS_PER_WAVE], l[ROWS_PER_WAVE], acc[ROWS_PER_WAVE][MAX_VCHUNKS], factor[ROWS_PER_WAVE];
    int pos[ROWS_PER_WAVE], head[ROWS_PER_WAVE], lo[ROWS_PER_WAVE];
    bool valid[ROWS_PER_WAVE];
#pragma unroll
    for (int rr = 0; rr < ROWS_PER_WAVE; ++rr) {
        const int r = wave * ROWS_PER_WAVE + rr;
        valid[rr] = r < n_rows;
        pos[rr] = first_pos + (valid[rr] ? r / heads_here : 0);
        head[rr] = head0 + (valid[rr] ? r % heads_here : 0);
        lo[rr] = first_seen(pos[rr], window, form.chunk);
        const int steps = temp_every > 0 ? (pos[rr] + 1) / temp_every : 0;
        factor[rr] = scale * (1.0f + temp_coef * logf(static_cast<float>(steps) + 1.0f));
        m[rr] = -INFINITY;
        l[rr] = 0.f;
#pragma unroll
        for (int cc = 0; cc < MAX_VCHUNKS; ++cc) acc[rr][cc] = 0.f;
    }
    const int last_pos = first_pos + n_tok - 1;
    const KeyWalk walk(first_pos, last_pos, window, keep_first, form.chunk);
    const int per_run = (walk.steps + n_runs - 1) / n_runs;                        // tiles of 64 keys a run
    const int v_end = std::min(walk.steps, (run + 1) * per_run);
    const int k_last = last_pos;
    const int32_t* table = block_table + static_cast<size_t>(seq) * table_width;
    for (int v = run * per_run; v < v_end; ++v) {
        const int k0 = walk.first_key(v);
        __syncthreads();                          // the tile before this one has been used by everyone
        stage_tile<T>(kpool, vpool, Ks, dkp, dk, k_row, Vs, dv, dv, table, page_size, kv_heads, kv, k0, k_last, k_pieces, v_pieces);
        __syncthreads();
        // scores of this lane's key for the wavefront's rows
        float s[ROWS_PER_WAVE];
#pragma unroll
        for (int rr = 0; rr < ROWS_PER_WAVE; ++rr) s[rr] = 0.f;
        const float* krow = Ks + lane * dkp;
        const float* qrow = Qs + wave * ROWS_PER_WAVE * dk;
        if (dkp == dk + 4) {
            for (int c = 0; c < dk; c += 4) {
                const float4 kv = *reinterpret_cast<const float4*>(krow + c);
#pragma unroll
                for (int rr = 0; rr < ROWS_PER_WAVE; ++rr) {
                    const float4 q = *reinterpret_cast<const float4*>(qrow + rr * dk + c);
                    s[rr] += q.x * kv.x + q.y * kv.y + q.z * kv.z + q.w * kv.w;
                }
            }
        } else {
            for (int c = 0; c < dk; ++c) {
                const float kv = krow[c];
#pragma unroll
                for (int rr = 0; rr < ROWS_PER_WAVE; ++rr) s[rr] += qrow[rr * dk + c] * kv;
            }
        }
        const int key = k0 + lane;
        float* prow = Ps + wave * ROWS_PER_WAVE * KEYS;
        float alpha[ROWS_PER_WAVE];
#pragma unroll
        for (int rr = 0; rr < ROWS_PER_WAVE; ++rr) {
            alpha[rr] = 1.f;
            if (!valid[rr]) { prow[rr * KEYS + lane] = 0.f; continue; }          // the same for the whole wavefront
            if (k0 > pos[rr]) { prow[rr * KEYS + lane] = 0.f; continue; }        // the same for the whole wavefront
            const bool seen = key_seen(key, pos[rr], lo[rr], keep_first);
            float sc = -INFINITY;
            if (seen) {
                const int back = std::min(pos[rr] - key, distances - 1);
                sc = s[rr] * factor[rr] + (bias ? bias[static_cast<size_t>(back) * H + head[rr]] : 0.f);
                if (form.softcap > 0.f) sc = soft_capped(sc, form.softcap, inv_cap);
            }
            const float m_new = fmaxf(m[rr], wave_max(sc));
            if (m_new == -INFINITY) { prow[rr * KEYS + lane] = 0.f; continue; }   // no key of this row so far (a window that starts later)
            alpha[rr] = expf(m[rr] - m_new);                      // 0 at the row's first keys
            const float p = seen ? expf(sc - m_new) : 0.f;
            l[rr] = l[rr] * alpha[rr] + wave_sum(p);
            m[rr] = m_new;
            prow[rr * KEYS + lane] = p;
        }
        // a wavefront reads only what it wrote itself: no barrier of the workgroup is needed here
        __builtin_amdgcn_wave_barrier();
#pragma unroll
        for (int cc = 0; cc < MAX_VCHUNKS; ++cc) {
            const int c = lane + cc * WAVE;
            if (c < dv) {
                float add[ROWS_PER_WAVE];
#pragma unroll
                for (int rr = 0; rr < ROWS_PER_WAVE; ++rr) add[rr] = 0.f;
                for (int j = 0; j < KEYS; j += 4) {
                    const float v0 = Vs[j * dv + c], v1 = Vs[(j + 1) * dv + c], v2 = Vs[(j + 2) * dv + c], v3 = Vs[(j + 3) * dv + c];
#pragma unroll
                    for (int rr = 0; rr < ROWS_PER_WAVE; ++rr) {
                        const float4 p = *reinterpret_cast<const float4*>(prow + rr * KEYS + j);
                        add[rr] += p.x * v0 + p.y * v1 + p.z * v2 + p.w * v3;
                    }
                }
#pragma unroll
                for (int rr = 0; rr < ROWS_PER_WAVE; ++rr) acc[rr][cc] = acc[rr][cc] * alpha[rr] + add[rr];
            }
        }
    }
#pragma unroll
    for (int rr = 0; rr < ROWS_PER_WAVE; ++rr) {
        if (!valid[rr]) continue;
        const int r = wave * ROWS_PER_WAVE + rr;
        if (partial) {
            float* prow = partial + ((static_cast<size_t>(first_row + r / heads_here) * H + head[rr]) * n_runs + run) * (dv + 2);
            if (lane == 0) { prow[0] = m[rr]; prow[1] = l[rr]; }
#pragma unroll
            for (int cc = 0; cc < MAX_VCHUNKS; ++cc) {
                const int c = lane + cc * WAVE;
                if (c < dv) prow[2 + c] = acc[rr][cc];
            }
            continue;
        }
        T* orow = out + static_cast<size_t>(first_row + r / heads_here) * (H * dv) + head[rr] * dv;
        float inv = out_scale / l[rr];
        if (sink) {             // one more term in the denominator: with M = max(m, sink), l e^(m - M) + e^(sink - M)
            const float sk = sink[head[rr]], M = fmaxf(m[rr], sk), w = expf(m[rr] - M);
            inv = out_scale * w / (l[rr] * w + expf(sk - M));
        }
#pragma unroll
        for (int cc = 0; cc < MAX_VCHUNKS; ++cc) {
            const int c = lane + cc * WAVE;
            if (c < dv) st(orow + c, acc[rr][cc] * inv * gate.of(first_row + r / heads_here, head[rr] * dv + c));
        }
    }
}

// ------------------------------------------------------------------ prompt portions on the matrix cores, in float32
// The same attention for tiles of up to 64 rows of (token, head), sixteen a wavefront, with both products on
// v_mfma_f32_16x16x4_f32 (true 32-bit products and sums; keys, values and queries are widened to float32 when they
// are staged).  Key and value sizes are multiples of 16.
//
//   S^T[key, row]  = K[key, :] . Q[row, :]    K rows as the first operand, Q rows as the second.  The k index of
//                    an MFMA is only a label: lane group kg (lane / 16) of step t takes channel kg dk/4 + t, so
//                    a lane reads dk/4 consecutive floats of its key and of its row.  A lane ends up with the
//                    scores of ONE row (lane % 16) for keys 16 j + 4 kg + r: bias, temperature and the running
//                    softmax are per lane, the row's maximum and sum cross the four lane groups only.
//   O^T[dim, row] += V^T[dim, key] . P^T[key, row]   the weight of key 16 j + 4 kg + r is register (j, r) of the
//                    lane, which is where the second operand of the MFMA over keys {16 j + 4 kg + r} wants it:
//                    the weights never leave the registers.  The lane holds dims 16 db + 4 kg + r of its row.
#define MROWS 64
typedef float floatx4_t __attribute__((ext_vector_type(4)));

// floats of the first region of the kernel's staging memory: the queries [MROWS][dk + 4], whose place the tiles of values
// [KEYS][dv + 4] take once the queries are in registers (no tile of values where keys and values are one pool)
__host__ __device__ __forceinline__ size_t mfma_first_floats(int dk, int dv, bool one_pool) {
    const size_t q = static_cast<size_t>(MROWS) * (dk + 4), v = one_pool ? 0 : static_cast<size_t>(KEYS) * (dv + 4);
    return q > v ? q : v;
}

__device__ __forceinline__ float groups4(float x, bool take_max) {
    // over the four lanes that hold one row (lanes r, r + 16, r + 32, r + 48): maximum or sum
    const auto a = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
    const float u = __uint_as_float(a[0]), v = __uint_as_float(a[1]);
    x = take_max ? fmaxf(u, v) : u + v;
    const auto b = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false, false);
    const float s = __uint_as_float(b[0]), t = __uint_as_float(b[1]);
    return take_max ? fmaxf(s, t) : s + t;
}

// QS: 16-byte pieces of a lane's quarter of a query row at most (dk <= 64 QS); DVB: blocks of 16 value channels at most
// (dv <= 16 DVB).  Both size arrays of registers, so the kernel is compiled for a few pairs of them.
template <typename T, int QS, int DVB>
__global__ void __launch_bounds__(WAVES * WAVE)
bias_attention_mfma_kernel(const T* __restrict__ qkv, int row_stride, const T* __restrict__ kpool, const T* __restrict__ vpool,
                           const int32_t* __restrict__ block_table, int table_width, const int32_t* __restrict__ tiles,
                           const int32_t* __restrict__ positions, const float* __restrict__ bias, int distances,
                           T* __restrict__ out, int H, int G, int dk, int dv, int page_size, float scale, float temp_coef,
                           int temp_every, int heads_per_chunk, bool k_pieces, bool v_pieces, int window, int keep_first,
                           float out_scale, const float* __restrict__ sink, ScoreForm form, float* __restrict__ partial, Gate gate) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int dkp = dk + 4, dvp = dv + 4;         // strides that spread the sixteen rows of a read over the banks
    // keys and values that are one pool (dv = dk) are staged once: the values are read from the keys' tile
    const bool one_pool = static_cast<const void*>(kpool) == static_cast<const void*>(vpool) && dk == dv;
    // the queries are staged once and then live in registers, a lane's quarter of its row; the tiles of values take
    // their place in LDS
    float* Qs = lds;                              // [MROWS][dkp], later [KEYS][dvp]
    float* Ks = lds + mfma_first_floats(dk, dv, one_pool);      // [KEYS][dkp]
    float* Vs = one_pool ? Ks : lds;
    const int tile = blockIdx.x, g = blockIdx.y, chunk = blockIdx.z;
    const int seq = tiles[4 * tile], first_row = tiles[4 * tile + 1], n_tok = tiles[4 * tile + 2];
    const int first_pos = positions[first_row];
    const int group = H / G;
    const int heads_here = std::min(heads_per_chunk, group - chunk * heads_per_chunk);
    const int head0 = g * group + chunk * heads_per_chunk;
    const int n_rows = n_tok * heads_here;        // row r = token r / heads_here, head r % heads_here
    const int tid = threadIdx.x, lane = tid & (WAVE - 1), wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
    const int i = lane & 15, kg = lane >> 4;
    const int kv = g / form.maps, kv_heads = G / form.maps, k_row = form.maps * dk;      // as in the kernel above
    kpool += (g % form.maps) * dk;
    const float inv_cap = form.softcap > 0.f ? 1.0f / form.softcap : 0.f;

    for (int e = tid; e < MROWS * dk; e += blockDim.x) {
        const int r = e / dk, c = e % dk;
        float v = 0.f;
        if (r < n_rows)
            v = ld(qkv + static_cast<size_t>(first_row + r / heads_here) * row_stride + (head0 + r % heads_here) * dk + c);
        Qs[r * dkp + c] = v;
    }
    const int row = wave * 16 + i;
    const bool valid = row < n_rows;
    const int pos = first_pos + (valid ? row / heads_here : 0);
    const int head = head0 + (valid ? row % heads_here : 0);
    const int lo = first_seen(pos, window, form.chunk);
    const int steps = temp_every > 0 ? (pos + 1) / temp_every : 0;
    const float factor = scale * (1.0f + temp_coef * logf(static_cast<float>(steps) + 1.0f));
    // the last position any row of this wavefront has (the same for all its lanes)
    const int wave_rows = std::min(16, n_rows - wave * 16);
    const int wave_last = wave_rows > 0 ? first_pos + (wave * 16 + wave_rows - 1) / heads_here : -1;
    float m = -INFINITY, l = 0.f;
    floatx4_t acc[DVB];                           // dv / 16 blocks of [4 dims] of the lane's row
#pragma unroll
    for (int db = 0; db < DVB; ++db) acc[db] = floatx4_t{0.f, 0.f, 0.f, 0.f};
    const int dvb = dv / 16, qsteps = dk / 16;    // value blocks; 16-byte reads of a lane's quarter of a row
    const int last_pos = first_pos + n_tok - 1;
    const int32_t* table = block_table + static_cast<size_t>(seq) * table_width;
    const float* qrow = Qs + row * dkp + kg * (dk / 4);
    __syncthreads();                              // the queries are all there
    float4 qreg[QS];
#pragma unroll
    for (int t4 = 0; t4 < QS; ++t4)
        qreg[t4] = t4 < qsteps ? *reinterpret_cast<const float4*>(qrow + 4 * t4) : make_float4(0.f, 0.f, 0.f, 0.f);
    const KeyWalk walk(first_pos, last_pos, window, keep_first, form.chunk);
    for (int v = 0; v < walk.steps; ++v) {
        const int k0 = walk.first_key(v);
        __syncthreads();                          // the tile before this one has been used by everyone
        // one after the other: both in registers at once would cost this kernel its second wavefront a SIMD
        stage_rows<T>(kpool, Ks, dkp, dk, k_row, table, page_size, kv_heads, kv, k0, last_pos, k_pieces);
        if (!one_pool) stage_rows<T>(vpool, Vs, dvp, dv, dv, table, page_size, kv_heads, kv, k0, last_pos, v_pieces);
        __syncthreads();
        if (k0 > wave_last) continue;             // nothing here for this wavefront's rows (it still stages and waits)
        floatx4_t sc[KEYS / 16];
#pragma unroll
        for (int j = 0; j < KEYS / 16; ++j) sc[j] = floatx4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t4 = 0; t4 < QS; ++t4) {
            if (t4 < qsteps) {
                const float4 qv = qreg[t4];
#pragma unroll
                for (int j = 0; j < KEYS / 16; ++j) {
                    const float4 kv = *reinterpret_cast<const float4*>(Ks + (16 * j + i) * dkp + kg * (dk / 4) + 4 * t4);
                    sc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(kv.x, qv.x, sc[j], 0, 0, 0);
                    sc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(kv.y, qv.y, sc[j], 0, 0, 0);
                    sc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(kv.z, qv.z, sc[j], 0, 0, 0);
                    sc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(kv.w, qv.w, sc[j], 0, 0, 0);
                }
            }
        }
        float top = -INFINITY;
#pragma unroll
        for (int j = 0; j < KEYS / 16; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int key = k0 + 16 * j + 4 * kg + r;
                float v = -INFINITY;
                if (valid && key_seen(key, pos, lo, keep_first)) {
                    const int back = std::min(pos - key, distances - 1);
                    v = sc[j][r] * factor + (bias ? bias[static_cast<size_t>(back) * H + head] : 0.f);
                    if (form.softcap > 0.f) v = soft_capped(v, form.softcap, inv_cap);
                }
                sc[j][r] = v;
                top = fmaxf(top, v);
            }
        top = groups4(top, true);
        const float m_new = fmaxf(m, top);
        const bool any = m_new > -INFINITY;       // a row that is no row, or whose keys all lie ahead, sees nothing
        const float alpha = any ? expf(m - m_new) : 1.f;          // 0 at the row's first keys
        float sum = 0.f;
#pragma unroll
        for (int j = 0; j < KEYS / 16; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const float p = any ? expf(sc[j][r] - m_new) : 0.f;           // e^-inf = 0 for a key that is not seen
                sc[j][r] = p;
                sum += p;
            }
        l = l * alpha + groups4(sum, false);
        m = m_new;
#pragma unroll
        for (int db = 0; db < DVB; ++db) {
            if (db < dvb) {
                floatx4_t a = acc[db] * alpha;
#pragma unroll
                for (int j = 0; j < KEYS / 16; ++j)
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        a = __builtin_amdgcn_mfma_f32_16x16x4f32(Vs[(16 * j + 4 * kg + r) * dvp + 16 * db + i], sc[j][r], a, 0, 0, 0);
                acc[db] = a;
            }
        }
    }
    if (!valid) return;
    if (partial) {              // an unfinished row, as the kernel above leaves a run of one
        float* prow = partial + (static_cast<size_t>(first_row + row / heads_here) * H + head) * (dv + 2);
        if (kg == 0) { prow[0] = m; prow[1] = l; }
#pragma unroll
        for (int db = 0; db < DVB; ++db) {
            if (db < dvb) {
#pragma unroll
                for (int r = 0; r < 4; r += 2)
                    *reinterpret_cast<float2*>(prow + 2 + 16 * db + 4 * kg + r) = make_float2(acc[db][r], acc[db][r + 1]);
            }
        }
        return;
    }
    T* orow = out + static_cast<size_t>(first_row + row / heads_here) * (H * dv) + head * dv + 4 * kg;
    float inv = out_scale / l;
    if (sink) {                 // one more term in the denominator: with M = max(m, sink), l e^(m - M) + e^(sink - M)
        const float sk = sink[head], M = fmaxf(m, sk), w = expf(m - M);
        inv = out_scale * w / (l * w + expf(sk - M));
    }
#pragma unroll
    for (int db = 0; db < DVB; ++db) {
        if (db < dvb) {
#pragma unroll
            for (int r = 0; r < 4; ++r)
                st(orow + 16 * db + r, acc[db][r] * inv * gate.of(first_row + row / heads_here, head * dv + 16 * db + 4 * kg + r));
        }
    }
}

// ------------------------------------------------------------------ prompt portions in bfloat16
// The same tiles for bfloat16 queries, keys and values, whose products are exact in float32 already: the scores are
// v_mfma_f32_16x16x32_bf16 sums, and a float32 weight goes into the second product as two bfloat16 numbers, its upper half
// as it stands and what that leaves, rounded (together the weight to 2^-16 of itself, far below the rounding of the values
// it meets).  Scores, cap, softmax and sums are float32, exponentials the hardware's exp2.
//
//   S^T[key, row]  = K . Q^T     lane (i, kg) gives 8 channels 32 kk + 8 kg.. of key i and of row i, and ends up with the
//                    scores of row i for keys 16 j + 4 kg + r
//   O^T[dim, row] += V^T . P^T   over 32 keys at a time: the k index of a lane's eight numbers is key 4 kg + e of either
//                    sixteen, where its own scores are; V^T is read from the tile [key][channel] by transposing reads
//
// A workgroup asks for the next tile's keys and values before it works on this one.  KQ: 32-channel pieces of a key, DVB:
// blocks of 16 value channels, at most; the registers are held to what lets two to four wavefronts share a SIMD, where the
// sizes allow (left alone the compiler takes accumulation registers besides, and one wavefront fewer fits: 176 instead of
// 128 us at keys of 64 and values of 128 channels).
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef short shortx4_t __attribute__((ext_vector_type(4)));
#define TILE_PAD 8             // elements of padding of a staged row: the rows of a read fall on different banks

// V^T for a 32-key product: gfx950's transposing read hands lane (i, kg) V[4 kg + e][dim0 + i], e = 0..3, when it gives the
// address of V[4 kg + i / 4][dim0 + 4 (i % 4)]; the second read takes the next sixteen keys
__device__ __forceinline__ bf16x8_t read_values_t(const uint16_t* tile, int row_elems, int dim0, int i, int kg) {
    typedef __attribute__((address_space(3))) shortx4_t* lds_ptr;
    const uint16_t* at = tile + (4 * kg + (i >> 2)) * row_elems + dim0 + 4 * (i & 3);
    const uint2 a = __builtin_bit_cast(uint2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)(at)));
    const uint2 b = __builtin_bit_cast(uint2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)(at + 16 * row_elems)));
    return __builtin_bit_cast(bf16x8_t, make_uint4(a.x, a.y, b.x, b.y));
}

template <int KQ, int DVB>
__global__ void __launch_bounds__(WAVES * WAVE, KQ > 4 ? 1 : DVB == 4 ? 4 - KQ / 4 : DVB == 8 ? 3 : 2)
bias_attention_bf16_kernel(const bf16_t* __restrict__ qkv, int row_stride, const bf16_t* __restrict__ kpool, const bf16_t* __restrict__ vpool,
                           const int32_t* __restrict__ block_table, int table_width, const int32_t* __restrict__ tiles,
                           const int32_t* __restrict__ positions, const float* __restrict__ bias, int distances, bf16_t* __restrict__ out,
                           int H, int G, int dk, int dv, int page_size, float scale, float temp_coef, int temp_every, int heads_per_chunk,
                           int window, int keep_first, float out_scale, const float* __restrict__ sink, ScoreForm form,
                           float* __restrict__ partial, Gate gate) {
    constexpr float LOG2E = 1.4426950408889634f, LN2 = 0.6931471805599453f;
    constexpr int KROW = 32 * KQ + TILE_PAD, VROW = 16 * DVB + TILE_PAD, VP = DVB / 2;
    __shared__ __attribute__((aligned(16))) uint16_t Ks[KEYS * KROW];
    __shared__ __attribute__((aligned(16))) uint16_t Vs[KEYS * VROW];
    const int tile = blockIdx.x, g = blockIdx.y, chunk = blockIdx.z;
    const int seq = tiles[4 * tile], first_row = tiles[4 * tile + 1], n_tok = tiles[4 * tile + 2];
    const int first_pos = positions[first_row];
    const int group = H / G;
    const int heads_here = std::min(heads_per_chunk, group - chunk * heads_per_chunk);
    const int head0 = g * group + chunk * heads_per_chunk;
    const int n_rows = n_tok * heads_here;        // row r = token r / heads_here, head r % heads_here
    const int tid = threadIdx.x, lane = tid & (WAVE - 1), wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
    const int i = lane & 15, kg = lane >> 4;
    const int kv = g / form.maps, kv_heads = G / form.maps, k_row = form.maps * dk;
    kpool += (g % form.maps) * dk;

    const int row = wave * 16 + i;
    const bool valid = row < n_rows;
    const int token = valid ? row / heads_here : 0;
    const int pos = first_pos + token;
    const int head = head0 + (valid ? row % heads_here : 0);
    const int lo = first_seen(pos, window, form.chunk);
    const int steps = temp_every > 0 ? (pos + 1) / temp_every : 0;
    const float factor = scale * (1.0f + temp_coef * logf(static_cast<float>(steps) + 1.0f));
    // a capped score, in units of log2: cap log2e tanh(s / cap) = c - 2 c / (2^(s 2 log2e / cap) + 1)
    const float cap2 = form.softcap * LOG2E, cap_in = form.softcap > 0.f ? 2.0f * LOG2E / form.softcap : 0.f;
    uint4 qf[KQ];
#pragma unroll
    for (int kk = 0; kk < KQ; ++kk) {
        const int c = 32 * kk + 8 * kg;
        qf[kk] = valid && c < dk ? *reinterpret_cast<const uint4*>(qkv + static_cast<size_t>(first_row + token) * row_stride + head * dk + c)
                                 : make_uint4(0u, 0u, 0u, 0u);
    }
    // the positions between which every row of this wavefront lies, and the last row's first key (the same for all its lanes)
    const int wave_rows = std::min(16, n_rows - wave * 16);
    const int wave_first = first_pos + (wave * 16) / heads_here;
    const int wave_last = wave_rows > 0 ? first_pos + (wave * 16 + wave_rows - 1) / heads_here : -1;
    const int wave_lo = first_seen(wave_last, window, form.chunk);
    float m = -INFINITY, l = 0.f;                 // the maximum in units of log2
    floatx4_t acc[DVB];
#pragma unroll
    for (int db = 0; db < DVB; ++db) acc[db] = floatx4_t{0.f, 0.f, 0.f, 0.f};
    const int dvb = dv / 16;
    const int last_pos = first_pos + n_tok - 1;
    const int32_t* table = block_table + static_cast<size_t>(seq) * table_width;
    const int k_pieces = dk / 8, v_pieces = dv / 8;
    uint4 kr[KQ], vr[VP];
    auto ask_pool = [&](const bf16_t* pool, int pieces, int row_elems, int k0, auto& regs, auto count) {
#pragma unroll
        for (int u = 0; u < decltype(count)::value; ++u) {
            const int idx = u * (WAVES * WAVE) + tid, j = idx / pieces, key = k0 + j;
            regs[u] = make_uint4(0u, 0u, 0u, 0u);
            if (j < KEYS && key <= last_pos) {
                const int page = table[key / page_size];
                if (page >= 0)
                    regs[u] = *reinterpret_cast<const uint4*>(pool + ((static_cast<size_t>(page) * kv_heads + kv) * page_size + key % page_size) *
                                                                         row_elems + (idx - j * pieces) * 8);
            }
        }
    };
    auto put_tile = [&](uint16_t* dst, int row_elems, int pieces, const auto& regs, auto count) {
#pragma unroll
        for (int u = 0; u < decltype(count)::value; ++u) {
            const int idx = u * (WAVES * WAVE) + tid, j = idx / pieces;
            if (j < KEYS) *reinterpret_cast<uint4*>(dst + j * row_elems + (idx - j * pieces) * 8) = regs[u];
        }
    };
    using KCount = std::integral_constant<int, KQ>;
    using VCount = std::integral_constant<int, VP>;
    if (dk < 32 * KQ) {                           // the channels that no key has meet zeros of the queries: they must be numbers
        for (int e = tid; e < KEYS * (32 * KQ - dk); e += WAVES * WAVE) Ks[e / (32 * KQ - dk) * KROW + dk + e % (32 * KQ - dk)] = 0;
    }
    const KeyWalk walk(first_pos, last_pos, window, keep_first, form.chunk);
    ask_pool(kpool, k_pieces, k_row, walk.first_key(0), kr, KCount{});
    ask_pool(vpool, v_pieces, dv, walk.first_key(0), vr, VCount{});
    for (int v = 0; v < walk.steps; ++v) {
        const int k0 = walk.first_key(v);
        __syncthreads();                          // the tile before this one has been used by everyone
        put_tile(Ks, KROW, k_pieces, kr, KCount{});
        put_tile(Vs, VROW, v_pieces, vr, VCount{});
        __syncthreads();
        if (v + 1 < walk.steps) {
            ask_pool(kpool, k_pieces, k_row, walk.first_key(v + 1), kr, KCount{});
            ask_pool(vpool, v_pieces, dv, walk.first_key(v + 1), vr, VCount{});
        }
        if (k0 > wave_last) continue;             // nothing here for this wavefront's rows (it still stages and waits)
        floatx4_t sc[KEYS / 16];
#pragma unroll
        for (int j = 0; j < KEYS / 16; ++j) {
            sc[j] = floatx4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < KQ; ++kk)
                if (32 * kk < dk)
                    sc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                        __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const uint4*>(Ks + (16 * j + i) * KROW + 32 * kk + 8 * kg)),
                        __builtin_bit_cast(bf16x8_t, qf[kk]), sc[j], 0, 0, 0);
        }
        float top = -INFINITY;
#pragma unroll
        for (int j = 0; j < KEYS / 16; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                float s = sc[j][r] * factor;
                if (bias) {
                    const int back = std::min(std::max(pos - (k0 + 16 * j + 4 * kg + r), 0), distances - 1);
                    s += bias[static_cast<size_t>(back) * H + head];
                }
                s = form.softcap > 0.f ? cap2 - 2.0f * cap2 * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s * cap_in) + 1.0f) : s * LOG2E;
                sc[j][r] = s;
            }
        if (k0 + KEYS - 1 > wave_first || k0 < wave_lo) {      // some row of this wavefront does not see every key of the tile
#pragma unroll
            for (int j = 0; j < KEYS / 16; ++j)
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (!key_seen(k0 + 16 * j + 4 * kg + r, pos, lo, keep_first)) sc[j][r] = -INFINITY;
        }
#pragma unroll
        for (int j = 0; j < KEYS / 16; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) top = fmaxf(top, sc[j][r]);
        top = groups4(top, true);
        const float m_new = fmaxf(m, top);
        const float m_ref = m_new > -INFINITY ? m_new : 0.f;   // a row whose keys all lie elsewhere: weights 2^-inf = 0
        const float alpha = __builtin_amdgcn_exp2f(m - m_ref); // 0 at the row's first keys
        float sum = 0.f;
        uint32_t hi[KEYS / 16][2], rest[KEYS / 16][2];         // the weights of a sixteen as pairs: upper halves, what they leave
#pragma unroll
        for (int j = 0; j < KEYS / 16; ++j)
#pragma unroll
            for (int r = 0; r < 4; r += 2) {
                const float p0 = __builtin_amdgcn_exp2f(sc[j][r] - m_ref), p1 = __builtin_amdgcn_exp2f(sc[j][r + 1] - m_ref);
                sum += p0 + p1;
                const uint32_t u0 = __float_as_uint(p0), u1 = __float_as_uint(p1);
                hi[j][r / 2] = (u0 >> 16) | (u1 & 0xffff0000u);
                rest[j][r / 2] = pack_bf16x2(p0 - __uint_as_float(u0 & 0xffff0000u), p1 - __uint_as_float(u1 & 0xffff0000u));
            }
        l = l * alpha + groups4(sum, false);
        m = m_new;
        const bool moved = __any(alpha != 1.f);                // no row's maximum rose: the sums stay as they are
#pragma unroll
        for (int db = 0; db < DVB; ++db) {
            if (db < dvb) {
                floatx4_t a = acc[db];
                if (moved) a = a * alpha;
#pragma unroll
                for (int jj = 0; jj < KEYS / 32; ++jj) {
                    const bf16x8_t vt = read_values_t(Vs + 32 * jj * VROW, VROW, 16 * db, i, kg);
                    a = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                        vt, __builtin_bit_cast(bf16x8_t, make_uint4(hi[2 * jj][0], hi[2 * jj][1], hi[2 * jj + 1][0], hi[2 * jj + 1][1])), a, 0, 0, 0);
                    a = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                        vt, __builtin_bit_cast(bf16x8_t, make_uint4(rest[2 * jj][0], rest[2 * jj][1], rest[2 * jj + 1][0], rest[2 * jj + 1][1])), a, 0, 0, 0);
                }
                acc[db] = a;
            }
        }
    }
    if (!valid) return;
    if (partial) {              // an unfinished row, as a run of one
        float* prow = partial + (static_cast<size_t>(first_row + token) * H + head) * (dv + 2);
        if (kg == 0) { prow[0] = m * LN2; prow[1] = l; }
#pragma unroll
        for (int db = 0; db < DVB; ++db) {
            if (db < dvb) {
#pragma unroll
                for (int r = 0; r < 4; r += 2)
                    *reinterpret_cast<float2*>(prow + 2 + 16 * db + 4 * kg + r) = make_float2(acc[db][r], acc[db][r + 1]);
            }
        }
        return;
    }
    float inv = out_scale / l;
    if (sink) {                 // one more term in the denominator, as in the kernels above
        const float sk = sink[head] * LOG2E, M = fmaxf(m, sk), w = __builtin_amdgcn_exp2f(m - M);
        inv = out_scale * w / (l * w + __builtin_amdgcn_exp2f(sk - M));
    }
    bf16_t* orow = out + static_cast<size_t>(first_row + token) * (H * dv) + head * dv + 4 * kg;
#pragma unroll
    for (int db = 0; db < DVB; ++db) {
        if (db < dvb) {
            float o[4] = {acc[db][0] * inv, acc[db][1] * inv, acc[db][2] * inv, acc[db][3] * inv};
            if (gate.rows) {
#pragma unroll
                for (int r = 0; r < 4; ++r) o[r] *= gate.of(first_row + token, head * dv + 16 * db + 4 * kg + r);
            }
            store_packed<bf16_t, 4>(orow + 16 * db, o);
        }
    }
}

// ------------------------------------------------------------------ single tokens and short portions in bfloat16
// The tiles of the vector-unit kernel (up to 16 rows of (token, head), one run of keys a workgroup) with the products of
// the kernel above.  Sixteen rows are one operand of an MFMA, so the four wavefronts share the run's keys instead of its
// rows: wavefront w takes the units of 32 keys w, w + 4, .., each with a maximum, sum and weighted sum of its own, which
// meet in LDS at the end.  Keys come from their pages straight into the first operand's registers (a lane: 8 channels of
// one key, 16 bytes); values go through a tile of the wavefront's own in LDS for the transposing reads, which needs no
// barrier.  The next unit's keys and values are asked for before the softmax of this one.
#define UNIT 32

template <int KQ, int DVB>
__global__ void __launch_bounds__(WAVES * WAVE)
bias_attention_bf16_token_kernel(const bf16_t* __restrict__ qkv, int row_stride, const bf16_t* __restrict__ kpool, const bf16_t* __restrict__ vpool,
                                 const int32_t* __restrict__ block_table, int table_width, const int32_t* __restrict__ tiles,
                                 const int32_t* __restrict__ positions, const float* __restrict__ bias, int distances, bf16_t* __restrict__ out,
                                 int H, int G, int dk, int dv, int page_size, float scale, float temp_coef, int temp_every, int heads_per_chunk,
                                 int n_runs, float* __restrict__ partial, int window, int keep_first, float out_scale,
                                 const float* __restrict__ sink, ScoreForm form, Gate gate) {
    constexpr float LOG2E = 1.4426950408889634f, LN2 = 0.6931471805599453f;
    constexpr int VROW = 16 * DVB + TILE_PAD, MROW = 16 * DVB;
    constexpr int TILE_BYTES = WAVES * UNIT * VROW * 2, MEET_BYTES = WAVES * ROWS * MROW * 4;
    __shared__ __attribute__((aligned(16))) unsigned char staged[TILE_BYTES > MEET_BYTES ? TILE_BYTES : MEET_BYTES];
    __shared__ float meet_m[WAVES][ROWS], meet_l[WAVES][ROWS];
    const int tile = blockIdx.x / n_runs, run = blockIdx.x % n_runs, g = blockIdx.y, chunk = blockIdx.z;
    const int seq = tiles[4 * tile], first_row = tiles[4 * tile + 1], n_tok = tiles[4 * tile + 2];
    const int first_pos = positions[first_row];
    const int group = H / G;
    const int heads_here = std::min(heads_per_chunk, group - chunk * heads_per_chunk);
    const int head0 = g * group + chunk * heads_per_chunk;
    const int n_rows = n_tok * heads_here;        // row r = token r / heads_here, head r % heads_here
    const int tid = threadIdx.x, lane = tid & (WAVE - 1), wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
    const int i = lane & 15, kg = lane >> 4;
    const int kv = g / form.maps, kv_heads = G / form.maps, k_row = form.maps * dk;
    kpool += (g % form.maps) * dk;
    uint16_t* Vs = reinterpret_cast<uint16_t*>(staged) + wave * UNIT * VROW;

    const bool valid = i < n_rows;
    const int token = valid ? i / heads_here : 0;
    const int pos = first_pos + token;
    const int head = head0 + (valid ? i % heads_here : 0);
    const int lo = first_seen(pos, window, form.chunk);
    const int steps = temp_every > 0 ? (pos + 1) / temp_every : 0;
    const float factor = scale * (1.0f + temp_coef * logf(static_cast<float>(steps) + 1.0f));
    const float cap2 = form.softcap * LOG2E, cap_in = form.softcap > 0.f ? 2.0f * LOG2E / form.softcap : 0.f;      // as in the kernel above
    uint4 qf[KQ];
#pragma unroll
    for (int kk = 0; kk < KQ; ++kk) {
        const int c = 32 * kk + 8 * kg;
        qf[kk] = valid && c < dk ? *reinterpret_cast<const uint4*>(qkv + static_cast<size_t>(first_row + token) * row_stride + head * dk + c)
                                 : make_uint4(0u, 0u, 0u, 0u);
    }
    float m = -INFINITY, l = 0.f;                 // of row i; the maximum in units of log2
    floatx4_t acc[DVB];
#pragma unroll
    for (int db = 0; db < DVB; ++db) acc[db] = floatx4_t{0.f, 0.f, 0.f, 0.f};
    const int dvb = dv / 16, v_pieces = dv / 8;
    const int last_pos = first_pos + n_tok - 1;
    const int last_lo = first_seen(last_pos, window, form.chunk);      // the latest first key of any row
    const int32_t* table = block_table + static_cast<size_t>(seq) * table_width;
    const KeyWalk walk(first_pos, last_pos, window, keep_first, form.chunk);
    const int per_run = (walk.steps + n_runs - 1) / n_runs;            // tiles of KEYS keys a run
    const int v0 = run * per_run, n_units = std::max(0, std::min(walk.steps, v0 + per_run) - v0) * (KEYS / UNIT);
    auto unit_key = [&](int u) { return walk.first_key(v0 + u / (KEYS / UNIT)) + u % (KEYS / UNIT) * UNIT; };
    uint4 kr[UNIT / 16][KQ], vr[DVB];
    auto page_of = [&](int key) { return key <= last_pos ? table[key / page_size] : -1; };
    auto ask = [&](int k0) {
#pragma unroll
        for (int j = 0; j < UNIT / 16; ++j) {
            const int key = k0 + 16 * j + i, page = page_of(key);
            const bf16_t* src = kpool + ((static_cast<size_t>(std::max(page, 0)) * kv_heads + kv) * page_size + key % page_size) * k_row + 8 * kg;
#pragma unroll
            for (int kk = 0; kk < KQ; ++kk)
                kr[j][kk] = page >= 0 && 32 * kk + 8 * kg < dk ? *reinterpret_cast<const uint4*>(src + 32 * kk) : make_uint4(0u, 0u, 0u, 0u);
        }
#pragma unroll
        for (int u = 0; u < DVB; ++u) {           // UNIT rows of v_pieces 16-byte pieces, a piece a lane: dv / 16 times
            vr[u] = make_uint4(0u, 0u, 0u, 0u);
            if (u < dvb) {
                const int idx = u * WAVE + lane, j = idx / v_pieces, key = k0 + j, page = page_of(key);
                if (page >= 0)
                    vr[u] = *reinterpret_cast<const uint4*>(vpool + ((static_cast<size_t>(page) * kv_heads + kv) * page_size + key % page_size) * dv +
                                                            (idx - j * v_pieces) * 8);
            }
        }
    };
    if (wave < n_units) ask(unit_key(wave));
    for (int u = wave; u < n_units; u += WAVES) {
        const int k0 = unit_key(u);
        floatx4_t sc[UNIT / 16];
#pragma unroll
        for (int j = 0; j < UNIT / 16; ++j) {
            sc[j] = floatx4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < KQ; ++kk)
                if (32 * kk < dk)
                    sc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, kr[j][kk]), __builtin_bit_cast(bf16x8_t, qf[kk]),
                                                                    sc[j], 0, 0, 0);
        }
        __builtin_amdgcn_wave_barrier();          // the reads of the unit before come first (one wavefront's LDS accesses stay in order)
#pragma unroll
        for (int x = 0; x < DVB; ++x) {
            if (x < dvb) {
                const int idx = x * WAVE + lane, j = idx / v_pieces;
                *reinterpret_cast<uint4*>(Vs + j * VROW + (idx - j * v_pieces) * 8) = vr[x];
            }
        }
        __builtin_amdgcn_wave_barrier();
        if (u + WAVES < n_units) ask(unit_key(u + WAVES));
        float top = -INFINITY;
#pragma unroll
        for (int j = 0; j < UNIT / 16; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                float s = sc[j][r] * factor;
                if (bias) {
                    const int back = std::min(std::max(pos - (k0 + 16 * j + 4 * kg + r), 0), distances - 1);
                    s += bias[static_cast<size_t>(back) * H + head];
                }
                sc[j][r] = form.softcap > 0.f ? cap2 - 2.0f * cap2 * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s * cap_in) + 1.0f) : s * LOG2E;
            }
        if (k0 + UNIT - 1 > first_pos || k0 < last_lo) {       // some row does not see every key of the unit
#pragma unroll
            for (int j = 0; j < UNIT / 16; ++j)
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (!key_seen(k0 + 16 * j + 4 * kg + r, pos, lo, keep_first)) sc[j][r] = -INFINITY;
        }
#pragma unroll
        for (int j = 0; j < UNIT / 16; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) top = fmaxf(top, sc[j][r]);
        top = groups4(top, true);
        const float m_new = fmaxf(m, top);
        const float m_ref = m_new > -INFINITY ? m_new : 0.f;   // a row that has seen no key yet: weights 2^-inf = 0
        const float alpha = __builtin_amdgcn_exp2f(m - m_ref); // 0 at the row's first keys
        float sum = 0.f;
        uint32_t hi[UNIT / 16][2], rest[UNIT / 16][2];         // the weights as pairs: upper halves, what they leave
#pragma unroll
        for (int j = 0; j < UNIT / 16; ++j)
#pragma unroll
            for (int r = 0; r < 4; r += 2) {
                const float p0 = __builtin_amdgcn_exp2f(sc[j][r] - m_ref), p1 = __builtin_amdgcn_exp2f(sc[j][r + 1] - m_ref);
                sum += p0 + p1;
                const uint32_t u0 = __float_as_uint(p0), u1 = __float_as_uint(p1);
                hi[j][r / 2] = (u0 >> 16) | (u1 & 0xffff0000u);
                rest[j][r / 2] = pack_bf16x2(p0 - __uint_as_float(u0 & 0xffff0000u), p1 - __uint_as_float(u1 & 0xffff0000u));
            }
        l = l * alpha + groups4(sum, false);
        m = m_new;
        const bf16x8_t p_hi = __builtin_bit_cast(bf16x8_t, make_uint4(hi[0][0], hi[0][1], hi[1][0], hi[1][1]));
        const bf16x8_t p_rest = __builtin_bit_cast(bf16x8_t, make_uint4(rest[0][0], rest[0][1], rest[1][0], rest[1][1]));
#pragma unroll
        for (int db = 0; db < DVB; ++db) {
            if (db < dvb) {
                const bf16x8_t vt = read_values_t(Vs, VROW, 16 * db, i, kg);
                floatx4_t a = acc[db] * alpha;
                a = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, p_hi, a, 0, 0, 0);
                acc[db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, p_rest, a, 0, 0, 0);
            }
        }
    }
    // the wavefronts' rows meet: a lane has dims 16 db + 4 kg .. of row i
    __syncthreads();
    float* meet = reinterpret_cast<float*>(staged);
#pragma unroll
    for (int db = 0; db < DVB; ++db)
        if (db < dvb)
            *reinterpret_cast<float4*>(meet + (wave * ROWS + i) * MROW + 16 * db + 4 * kg) = make_float4(acc[db][0], acc[db][1], acc[db][2], acc[db][3]);
    if (kg == 0) {
        meet_m[wave][i] = m;
        meet_l[wave][i] = l;
    }
    __syncthreads();
    for (int e = tid; e < n_rows * dv; e += WAVES * WAVE) {
        const int r = e / dv, c = e - r * dv, t = first_row + r / heads_here, hd = head0 + r % heads_here;
        float M = meet_m[0][r], L = 0.f, a = 0.f;
#pragma unroll
        for (int w = 1; w < WAVES; ++w) M = fmaxf(M, meet_m[w][r]);
        const float ref = M > -INFINITY ? M : 0.f;
#pragma unroll
        for (int w = 0; w < WAVES; ++w) {
            const float f = __builtin_amdgcn_exp2f(meet_m[w][r] - ref);
            L += f * meet_l[w][r];
            a += f * meet[(w * ROWS + r) * MROW + c];
        }
        if (partial) {
            float* prow = partial + ((static_cast<size_t>(t) * H + hd) * n_runs + run) * (dv + 2);
            if (c == 0) { prow[0] = M * LN2; prow[1] = L; }
            prow[2 + c] = a;
            continue;
        }
        float inv = out_scale / L;
        if (sink) {             // one more term in the denominator, as in the kernels above
            const float sk = sink[hd] * LOG2E, top = fmaxf(M, sk), f = __builtin_amdgcn_exp2f(M - top);
            inv = out_scale * f / (L * f + __builtin_amdgcn_exp2f(sk - top));
        }
        st(out + static_cast<size_t>(t) * (H * dv) + hd * dv + c, a * inv * gate.of(t, hd * dv + c));
    }
}

// out[row, :] = sum_r acc_r e^(m_r - M) / (sum_r l_r e^(m_r - M) + e^(sink - M)) over the runs of a row (an empty run
// has l = 0; no sink: no such term; M is the maximum over the runs and the sink).
// The weights e^(m_r - M) go through LDS, and the sums over the runs then read nothing that depends on an earlier read.
// One workgroup a row, of as many wavefronts as the row has runs of 64 value channels (up to four); every wavefront works
// the runs' weights out for itself (lane r takes run r's maximum and sum, n_runs <= 64) and sums its own channels.
template <typename T>
__global__ void __launch_bounds__(MAX_VCHUNKS * WAVE) merge_runs_kernel(const float* __restrict__ partial, T* __restrict__ out, int n_runs,
                                                                        int dv, float out_scale, const float* __restrict__ sink, int H, Gate gate) {
    __shared__ float weight[MAX_VCHUNKS][WAVE];
    const size_t row = blockIdx.x;
    const float* p = partial + row * n_runs * (dv + 2);
    const int lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE;
    float m = -INFINITY, l = 0.f;
    if (lane < n_runs) {
        m = p[lane * (dv + 2)];
        l = p[lane * (dv + 2) + 1];
    }
    if (!(l > 0.f)) m = -INFINITY;
    float M = wave_max(m);
    const float sk = sink ? sink[row % H] : -INFINITY;        // rows are (token, head); the sink counts once, here
    M = fmaxf(M, sk);
    const float w = l > 0.f ? expf(m - M) : 0.f;
    const float L = wave_sum(l * w) + (sink ? expf(sk - M) : 0.f);
    weight[wave][lane] = w;
    __builtin_amdgcn_wave_barrier();          // a wavefront reads only the weights it wrote itself
    for (int c = wave * WAVE + lane; c < dv; c += blockDim.x) {
        float a = 0.f;
        for (int r = 0; r < n_runs; ++r) {
            const float wr = weight[wave][r];
            if (wr > 0.f) a += p[r * (dv + 2) + 2 + c] * wr;
        }
        st(out + row * dv + c, a * out_scale / L * gate.of(row / H, static_cast<int>(row % H) * dv + c));
    }
}

// Differential heads: two maps of every head over the same values, o = a1 - lambda a2 (a1, a2 the maps' finished rows),
// o / sqrt(mean(o^2) + eps) over the head's channels, times out_scale.  `partial`: rows of (token, query head), the query
// heads in the order [kv head][map][head of the group], in n_runs runs each, as the kernels above leave them.
// One workgroup a (token, head), a wavefront for every 64 value channels.
template <typename T>
__global__ void __launch_bounds__(MAX_VCHUNKS * WAVE) merge_maps_kernel(const float* __restrict__ partial, T* __restrict__ out, int n_runs,
                                                                        int heads, int group, int dv, float lambda, float eps,
                                                                        float out_scale) {
    __shared__ float weight[MAX_VCHUNKS][2][WAVE];
    __shared__ float scratch[16];
    const int t = blockIdx.x / heads, h = blockIdx.x % heads;
    const int lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE;
    const size_t first = (static_cast<size_t>(t) * heads * 2 + static_cast<size_t>(h / group) * 2 * group + h % group) * n_runs * (dv + 2);
    const float* p[2] = {partial + first, partial + first + static_cast<size_t>(group) * n_runs * (dv + 2)};
#pragma unroll
    for (int k = 0; k < 2; ++k) {
        float m = -INFINITY, l = 0.f;
        if (lane < n_runs) {
            m = p[k][lane * (dv + 2)];
            l = p[k][lane * (dv + 2) + 1];
        }
        if (!(l > 0.f)) m = -INFINITY;
        const float M = wave_max(m);
        const float w = l > 0.f ? expf(m - M) : 0.f;
        const float L = wave_sum(l * w);
        weight[wave][k][lane] = (k == 0 ? w : -lambda * w) / L;
    }
    __builtin_amdgcn_wave_barrier();          // a wavefront reads only the weights it wrote itself
    const int c = wave * WAVE + lane;
    float o = 0.f;
    if (c < dv) {
        for (int r = 0; r < n_runs; ++r) {
            const float w1 = weight[wave][0][r], w2 = weight[wave][1][r];
            // (an empty run has written nothing but its maximum and sum of zeros worth: its weight is zero, its row finite)
            const float a1 = p[0][r * (dv + 2) + 2 + c], a2 = p[1][r * (dv + 2) + 2 + c];
            o += w1 * a1 + w2 * a2;
        }
    }
    const float r = out_scale / sqrtf(block_sum(o * o, scratch) / static_cast<float>(dv) + eps);
    if (c < dv) st(out + (static_cast<size_t>(t) * heads + h) * dv + c, o * r);
}

// The same for rows of one run and an even number of channels: a wavefront a (token, head), two neighbouring channels a
// lane and 128, nothing through LDS.
template <typename T>
__global__ void __launch_bounds__(256) merge_maps_one_kernel(const float* __restrict__ partial, T* __restrict__ out, int rows, int heads,
                                                             int group, int dv, float lambda, float eps, float out_scale) {
    const int row = blockIdx.x * (blockDim.x / WAVE) + threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
    if (row >= rows) return;
    const int t = row / heads, h = row % heads;
    const float* p1 = partial + (static_cast<size_t>(t) * heads * 2 + static_cast<size_t>(h / group) * 2 * group + h % group) * (dv + 2);
    const float* p2 = p1 + static_cast<size_t>(group) * (dv + 2);
    const float w1 = 1.0f / p1[1], w2 = lambda / p2[1];
    float2 o[MAX_VCHUNKS / 2];
    float ss = 0.f;
#pragma unroll
    for (int u = 0; u < MAX_VCHUNKS / 2; ++u) {
        const int c = 2 * lane + 2 * WAVE * u;
        o[u] = make_float2(0.f, 0.f);
        if (c < dv) {
            const float2 a1 = *reinterpret_cast<const float2*>(p1 + 2 + c), a2 = *reinterpret_cast<const float2*>(p2 + 2 + c);
            o[u] = make_float2(a1.x * w1 - a2.x * w2, a1.y * w1 - a2.y * w2);
            ss += o[u].x * o[u].x + o[u].y * o[u].y;
        }
    }
    const float r = out_scale / sqrtf(wave_sum(ss) / static_cast<float>(dv) + eps);
#pragma unroll
    for (int u = 0; u < MAX_VCHUNKS / 2; ++u) {
        const int c = 2 * lane + 2 * WAVE * u;
        if (c < dv) {
            T* dst = out + static_cast<size_t>(row) * dv + c;
            if constexpr (sizeof(T) == 2) *reinterpret_cast<uint32_t*>(dst) = pack_bf16x2(o[u].x * r, o[u].y * r);
            else *reinterpret_cast<float2*>(dst) = make_float2(o[u].x * r, o[u].y * r);
        }
    }
}

// partial float32 [T][2 heads][n_runs][dv + 2]; out [T][heads][dv] of the type `dtype`
NI_EXPORT int ni_merge_maps(const void* partial, void* out, int T, int heads, int kv_heads, int dv, int n_runs, float lambda, float eps,
                            float out_scale, int dtype, hipStream_t stream) {
    if (T <= 0) return 0;
    if (heads < 1 || kv_heads < 1 || heads % kv_heads || n_runs < 1 || n_runs > WAVE || dv < 1 || dv > MAX_VCHUNKS * WAVE) return -1;
    if (n_runs == 1 && dv % 2 == 0 && reinterpret_cast<uintptr_t>(partial) % 8 == 0 && reinterpret_cast<uintptr_t>(out) % 8 == 0) {
        const unsigned blocks = static_cast<unsigned>((static_cast<size_t>(T) * heads + 3) / 4);
        if (dtype == 0)
            merge_maps_one_kernel<float><<<blocks, 256, 0, stream>>>((const float*)partial, (float*)out, T * heads, heads, heads / kv_heads, dv,
                                                                     lambda, eps, out_scale);
        else
            merge_maps_one_kernel<bf16_t><<<blocks, 256, 0, stream>>>((const float*)partial, (bf16_t*)out, T * heads, heads, heads / kv_heads, dv,
                                                                      lambda, eps, out_scale);
        return NI_LAUNCH_RESULT();
    }
    const int threads = (dv + WAVE - 1) / WAVE * WAVE;
    if (dtype == 0)
        merge_maps_kernel<float><<<T * heads, threads, 0, stream>>>((const float*)partial, (float*)out, n_runs, heads, heads / kv_heads, dv,
                                                                    lambda, eps, out_scale);
    else
        merge_maps_kernel<bf16_t><<<T * heads, threads, 0, stream>>>((const float*)partial, (bf16_t*)out, n_runs, heads, heads / kv_heads, dv,
                                                                     lambda, eps, out_scale);
    return NI_LAUNCH_RESULT();
}

NI_EXPORT int ni_kv_store(const void* qkv, int row_stride, int k_off, int v_off, const void* slot_mapping, void* kpool,
                          void* vpool, int T, int G, int dk, int dv, int page_size, int dtype, hipStream_t stream) {
    if (T <= 0) return 0;
    if (dtype == 0)
        kv_store_kernel<float><<<T, 256, 0, stream>>>((const float*)qkv, row_stride, k_off, v_off, (const int32_t*)slot_mapping,
                                                      (float*)kpool, (float*)vpool, G, dk, dv, page_size);
    else
        kv_store_kernel<bf16_t><<<T, 256, 0, stream>>>((const bf16_t*)qkv, row_stride, k_off, v_off, (const int32_t*)slot_mapping,
                                                       (bf16_t*)kpool, (bf16_t*)vpool, G, dk, dv, page_size);
    return NI_LAUNCH_RESULT();
}

struct MfmaArgs {
    const void *qkv; int row_stride; const void *kpool, *vpool, *block_table; int table_width; const void *tiles, *positions, *bias;
    int distances; void* out; int H, G, dk, dv, page_size; float scale, temp_coef; int temp_every, heads_per_chunk;
    bool k_pieces, v_pieces; int window, keep_first; float out_scale; const void* sink; ScoreForm form; void* partial; Gate gate;
};

// Sizes that the kernel for single tokens and short portions in bfloat16 takes: rows of whole 16-byte pieces, values in blocks
// of 16 channels
static bool bf16_tokens(int dk, int dv) { return dk % 8 == 0 && dk >= 8 && dk <= 256 && dv % 16 == 0 && dv >= 16 && dv <= 256; }

NI_EXPORT int ni_bias_attention_bf16_tokens(int dk, int dv) { return bf16_tokens(dk, dv); }

template <int KQ, int DVB>
static void launch_tokens(const MfmaArgs& a, int n_runs, dim3 grid, hipStream_t stream) {
    bias_attention_bf16_token_kernel<KQ, DVB><<<grid, WAVES * WAVE, 0, stream>>>(
        (const bf16_t*)a.qkv, a.row_stride, (const bf16_t*)a.kpool, (const bf16_t*)a.vpool, (const int32_t*)a.block_table, a.table_width,
        (const int32_t*)a.tiles, (const int32_t*)a.positions, (const float*)a.bias, a.distances, (bf16_t*)a.out, a.H, a.G, a.dk, a.dv,
        a.page_size, a.scale, a.temp_coef, a.temp_every, a.heads_per_chunk, n_runs, (float*)a.partial, a.window, a.keep_first, a.out_scale,
        (const float*)a.sink, a.form, a.gate);
}

template <int KQ>
static void launch_tokens_values(const MfmaArgs& a, int n_runs, dim3 grid, hipStream_t stream) {
    if (a.dv <= 64) launch_tokens<KQ, 4>(a, n_runs, grid, stream);
    else if (a.dv <= 128) launch_tokens<KQ, 8>(a, n_runs, grid, stream);
    else launch_tokens<KQ, 16>(a, n_runs, grid, stream);
}

NI_EXPORT int ni_bias_attention_rows() { return ROWS; }

NI_EXPORT int ni_bias_attention(const void* qkv, int row_stride, const void* kpool, const void* vpool, const void* block_table,
                                int table_width, const void* tiles, int n_tiles, const void* positions, const void* bias, int distances, void* out,
                                int H, int G, int dk, int dv, int page_size, float scale, float temp_coef, int temp_every,
                                int heads_per_chunk, int n_runs, void* partial, int n_rows, int waves, int window, int keep_first,
                                float out_scale, const void* sink, float softcap, int chunk, int maps, int unfinished, const void* gate_rows,
                                int gate_stride, int gate_every, int dtype, hipStream_t stream) {
    // `unfinished`: the rows stay in `partial`, runs unmerged (also a single run), for a kernel that finishes them; no sink
    if (n_tiles <= 0) return 0;
    if (window < 0 || keep_first < 0 || chunk < 0 || (chunk && window) || maps < 1 || G % maps) return -1;
    if (unfinished && (!partial || sink || gate_rows)) return -1;
    if (gate_rows && (gate_every < 1 || gate_stride < (H * dv + gate_every - 1) / gate_every || maps != 1)) return -1;
    const Gate gate{(const float*)gate_rows, gate_stride, gate_every};
    const ScoreForm form{softcap, chunk, maps};
    if (dv > MAX_VCHUNKS * WAVE || H % G || heads_per_chunk < 1 || heads_per_chunk > ROWS) return -1;
    const int group = H / G;
    const int dkp = dk % 4 == 0 ? dk + 4 : dk + 1;
    const size_t lds = (static_cast<size_t>(ROWS) * dk + static_cast<size_t>(KEYS) * dkp + static_cast<size_t>(KEYS) * dv +
                        WAVES * ROWS_PER_WAVE * KEYS) * sizeof(float);
    if (lds > 160 * 1024) return -2;
    if (n_runs < 1 || (n_runs > 1 && !partial) || waves < 1 || waves > WAVES) return -1;
    const int vec = dtype == 0 ? 4 : 8;
    const bool k_pieces = dk % vec == 0 && reinterpret_cast<uintptr_t>(kpool) % 16 == 0;
    const bool v_pieces = dv % vec == 0 && reinterpret_cast<uintptr_t>(vpool) % 16 == 0;
    if (n_runs == 1 && !unfinished) partial = nullptr;
    dim3 grid(n_tiles * n_runs, G, (group + heads_per_chunk - 1) / heads_per_chunk);
    hipError_t err = hipSuccess;
    if (dtype == 0) {
        static size_t allowed = 48 * 1024;
        if (lds > allowed && (allowed = lds))
            err = hipFuncSetAttribute((const void*)bias_attention_kernel<float>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (err != hipSuccess) return (int)err;
        bias_attention_kernel<float><<<grid, waves * WAVE, lds, stream>>>(
            (const float*)qkv, row_stride, (const float*)kpool, (const float*)vpool, (const int32_t*)block_table, table_width,
            (const int32_t*)tiles, (const int32_t*)positions, (const float*)bias, distances, (float*)out, H, G, dk, dv, page_size, scale, temp_coef,
            temp_every, heads_per_chunk, n_runs, (float*)partial, k_pieces, v_pieces, dkp, window, keep_first, out_scale,
            (const float*)sink, form, gate);
        if (partial && !unfinished) merge_runs_kernel<float><<<n_rows * H, std::min(MAX_VCHUNKS, (dv + WAVE - 1) / WAVE) * WAVE, 0, stream>>>((const float*)partial, (float*)out, n_runs, dv, out_scale,
                                                                             (const float*)sink, H, gate);
    } else if (bf16_tokens(dk, dv) && k_pieces && v_pieces && row_stride % 8 == 0 && reinterpret_cast<uintptr_t>(qkv) % 16 == 0) {
        const MfmaArgs args{qkv, row_stride, kpool, vpool, block_table, table_width, tiles, positions, bias, distances, out, H, G, dk, dv,
                            page_size, scale, temp_coef, temp_every, heads_per_chunk, k_pieces, v_pieces, window, keep_first, out_scale, sink,
                            form, partial, gate};
        if (dk <= 32) launch_tokens_values<1>(args, n_runs, grid, stream);
        else if (dk <= 64) launch_tokens_values<2>(args, n_runs, grid, stream);
        else if (dk <= 128) launch_tokens_values<4>(args, n_runs, grid, stream);
        else launch_tokens_values<8>(args, n_runs, grid, stream);
        if (partial && !unfinished) merge_runs_kernel<bf16_t><<<n_rows * H, std::min(MAX_VCHUNKS, (dv + WAVE - 1) / WAVE) * WAVE, 0, stream>>>((const float*)partial, (bf16_t*)out, n_runs, dv, out_scale,
                                                                              (const float*)sink, H, gate);
    } else {
        static size_t allowed = 48 * 1024;
        if (lds > allowed && (allowed = lds))
            err = hipFuncSetAttribute((const void*)bias_attention_kernel<bf16_t>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (err != hipSuccess) return (int)err;
        bias_attention_kernel<bf16_t><<<grid, waves * WAVE, lds, stream>>>(
            (const bf16_t*)qkv, row_stride, (const bf16_t*)kpool, (const bf16_t*)vpool, (const int32_t*)block_table, table_width,
            (const int32_t*)tiles, (const int32_t*)positions, (const float*)bias, distances, (bf16_t*)out, H, G, dk, dv, page_size, scale, temp_coef,
            temp_every, heads_per_chunk, n_runs, (float*)partial, k_pieces, v_pieces, dkp, window, keep_first, out_scale,
            (const float*)sink, form, gate);
        if (partial && !unfinished) merge_runs_kernel<bf16_t><<<n_rows * H, std::min(MAX_VCHUNKS, (dv + WAVE - 1) / WAVE) * WAVE, 0, stream>>>((const float*)partial, (bf16_t*)out, n_runs, dv, out_scale,
                                                                              (const float*)sink, H, gate);
    }
    return NI_LAUNCH_RESULT();
}

// staging memory of the matrix-core kernel: the queries (then the tiles of values) and a tile of keys
static size_t mfma_lds_bytes(int dk, int dv, bool one_pool) {
    return (mfma_first_floats(dk, dv, one_pool) + static_cast<size_t>(KEYS) * (dk + 4)) * sizeof(float);
}

// rows of (token, head) of a tile of the matrix-core kernel; 0 where it does not take these sizes.  `one_pool`: keys
// and values are the same pool (dv = dk)
NI_EXPORT int ni_bias_attention_mfma_rows(int dk, int dv, int one_pool) {
    if (dk % 16 || dv % 16 || dk < 16 || dv < 16 || dv > MAX_VCHUNKS * WAVE || (one_pool && dk != dv)) return 0;
    return mfma_lds_bytes(dk, dv, one_pool != 0) <= 160 * 1024 ? MROWS : 0;
}

template <typename T, int QS, int DVB>
static hipError_t launch_mfma(const MfmaArgs& a, dim3 grid, size_t lds, hipStream_t stream) {
    static size_t allowed = 48 * 1024;            // of this instance of the kernel
    if (lds > allowed) {
        const hipError_t err = hipFuncSetAttribute((const void*)bias_attention_mfma_kernel<T, QS, DVB>,
                                                   hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (err != hipSuccess) return err;
        allowed = lds;
    }
    bias_attention_mfma_kernel<T, QS, DVB><<<grid, WAVES * WAVE, lds, stream>>>(
        (const T*)a.qkv, a.row_stride, (const T*)a.kpool, (const T*)a.vpool, (const int32_t*)a.block_table, a.table_width,
        (const int32_t*)a.tiles, (const int32_t*)a.positions, (const float*)a.bias, a.distances, (T*)a.out, a.H, a.G, a.dk, a.dv,
        a.page_size, a.scale, a.temp_coef, a.temp_every, a.heads_per_chunk, a.k_pieces, a.v_pieces, a.window, a.keep_first,
        a.out_scale, (const float*)a.sink, a.form, (float*)a.partial, a.gate);
    return hipSuccess;
}

template <int KQ, int DVB>
static void launch_bf16(const MfmaArgs& a, dim3 grid, hipStream_t stream) {
    bias_attention_bf16_kernel<KQ, DVB><<<grid, WAVES * WAVE, 0, stream>>>(
        (const bf16_t*)a.qkv, a.row_stride, (const bf16_t*)a.kpool, (const bf16_t*)a.vpool, (const int32_t*)a.block_table, a.table_width,
        (const int32_t*)a.tiles, (const int32_t*)a.positions, (const float*)a.bias, a.distances, (bf16_t*)a.out, a.H, a.G, a.dk, a.dv,
        a.page_size, a.scale, a.temp_coef, a.temp_every, a.heads_per_chunk, a.window, a.keep_first, a.out_scale, (const float*)a.sink, a.form,
        (float*)a.partial, a.gate);
}

template <int KQ>
static void launch_bf16_values(const MfmaArgs& a, dim3 grid, hipStream_t stream) {
    if (a.dv <= 64) launch_bf16<KQ, 4>(a, grid, stream);
    else if (a.dv <= 128) launch_bf16<KQ, 8>(a, grid, stream);
    else launch_bf16<KQ, 16>(a, grid, stream);
}

// tiles of up to 64 rows (tokens * heads of a chunk), no runs: for steps with portions of prompts
NI_EXPORT int ni_bias_attention_mfma(const void* qkv, int row_stride, const void* kpool, const void* vpool, const void* block_table,
                                     int table_width, const void* tiles, int n_tiles, const void* positions, const void* bias,
                                     int distances, void* out, int H, int G, int dk, int dv, int page_size, float scale,
                                     float temp_coef, int temp_every, int heads_per_chunk, int window, int keep_first,
                                     float out_scale, const void* sink, float softcap, int chunk, int maps, void* partial, const void* gate_rows,
                                     int gate_stride, int gate_every, int dtype, hipStream_t stream) {
    // `partial` (float32 [T][H][dv + 2], or null): the rows are left there unfinished, as runs of one; no sink
    if (n_tiles <= 0) return 0;
    if (window < 0 || keep_first < 0 || chunk < 0 || (chunk && window) || maps < 1 || G % maps || (partial && (sink || gate_rows))) return -1;
    if (gate_rows && (gate_every < 1 || gate_stride < (H * dv + gate_every - 1) / gate_every || maps != 1)) return -1;
    const bool one_pool = kpool == vpool && dk == dv;
    if (!ni_bias_attention_mfma_rows(dk, dv, one_pool) || H % G || heads_per_chunk < 1 || heads_per_chunk > MROWS) return -1;
    const int group = H / G;
    const size_t lds = mfma_lds_bytes(dk, dv, one_pool);
    const int vec = dtype == 0 ? 4 : 8;
    const bool k_pieces = dk % vec == 0 && reinterpret_cast<uintptr_t>(kpool) % 16 == 0;
    const bool v_pieces = dv % vec == 0 && reinterpret_cast<uintptr_t>(vpool) % 16 == 0;
    dim3 grid(n_tiles, G, (group + heads_per_chunk - 1) / heads_per_chunk);
    const MfmaArgs args{qkv, row_stride, kpool, vpool, block_table, table_width, tiles, positions, bias, distances, out, H, G, dk, dv,
                        page_size, scale, temp_coef, temp_every, heads_per_chunk, k_pieces, v_pieces, window, keep_first, out_scale, sink,
                        ScoreForm{softcap, chunk, maps}, partial, Gate{(const float*)gate_rows, gate_stride, gate_every}};
    hipError_t err;
    // bfloat16 rows in whole 16-byte pieces
    if (dtype == 1 && k_pieces && v_pieces && row_stride % 8 == 0 && reinterpret_cast<uintptr_t>(qkv) % 16 == 0) {
        if (dk <= 32) launch_bf16_values<1>(args, grid, stream);
        else if (dk <= 64) launch_bf16_values<2>(args, grid, stream);
        else if (dk <= 128) launch_bf16_values<4>(args, grid, stream);
        else launch_bf16_values<8>(args, grid, stream);
        return NI_LAUNCH_RESULT();
    }
    // the smallest arrays of registers that hold these sizes
    if (dk <= 64 && dv <= 64) err = dtype == 0 ? launch_mfma<float, 4, 4>(args, grid, lds, stream) : launch_mfma<bf16_t, 4, 4>(args, grid, lds, stream);
    else if (dk <= 128 && dv <= 64) err = dtype == 0 ? launch_mfma<float, 8, 4>(args, grid, lds, stream) : launch_mfma<bf16_t, 8, 4>(args, grid, lds, stream);
    else if (dk <= 128) err = dtype == 0 ? launch_mfma<float, 8, 16>(args, grid, lds, stream) : launch_mfma<bf16_t, 8, 16>(args, grid, lds, stream);
    else err = dtype == 0 ? launch_mfma<float, 16, 16>(args, grid, lds, stream) : launch_mfma<bf16_t, 16, 16>(args, grid, lds, stream);
    if (err != hipSuccess) return (int)err;
    return NI_LAUNCH_RESULT();
}
