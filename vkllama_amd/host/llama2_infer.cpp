// Command-line generation with the C++ classes, from a GGUF file or a folder with
// config.json and model.safetensors: the flow
// of the reference's app/llama2_infer.cpp (open the file, collect keys and
// tensors, Model::init, prompt pass, then one token per step picked on the
// host by a TopkSampler(1), line 138 there) without the sentencepiece
// tokenizer, which is not available to C++ in this image: the prompt is given
// as token ids.
//
//   llama2_infer [--topk K | --topp P] [--seed S] [--dtype bfloat16|float32]
//                [--max-tokens N] MODEL N_TOKENS ID [ID ...]
#include "models/registry.h"
#include "models/samplers.h"
#include <cstring>
#include <memory>
#include <algorithm>
#include <chrono>
#include <cstdio>
#include <cstdlib>
#include <map>
#include <string>
#include <vector>

int
main (int argc, char **argv)
{
  size_t topk = 1;
  float topp = -1.f;
  bool seeded = false;
  uint64_t seed = 0;
  vkllama::ModelOptions options;
  while (argc > 2 && argv[1][0] == '-' && argv[1][1] == '-')
    {
      if (!strcmp (argv[1], "--topk"))
        topk = (size_t)strtoul (argv[2], nullptr, 10);
      else if (!strcmp (argv[1], "--topp"))
        topp = strtof (argv[2], nullptr);
      else if (!strcmp (argv[1], "--seed"))
        seeded = true, seed = strtoull (argv[2], nullptr, 10);
      else if (!strcmp (argv[1], "--dtype") && (!strcmp (argv[2], "bfloat16") || !strcmp (argv[2], "float32")))
        options.dtype = argv[2][0] == 'f' ? vkllama::FP32 : vkllama::BF16;
      else if (!strcmp (argv[1], "--max-tokens"))
        options.max_tokens = strtoull (argv[2], nullptr, 10);
      else
        break;
      argv += 2, argc -= 2;
    }
  if (argc < 4 || topk < 1)
    {
      fprintf (stderr,
               "usage: llama2_infer [--topk K | --topp P] [--seed S] [--dtype bfloat16|float32] "
               "[--max-tokens N] <model> <predict tokens> "
               "<prompt id> [id ...]\n");
      return 2;
    }
  std::unique_ptr<Sampler> sampler;
  if (topp >= 0.f)
    sampler.reset (seeded ? new TopPSampler (topp, seed) : new TopPSampler (topp));
  else
    sampler.reset (seeded ? new TopkSampler (topk, seed) : new TopkSampler (topk));
  const int predict = atoi (argv[2]);
  std::vector<uint32_t> prompt;
  for (int i = 3; i < argc; ++i)
    prompt.push_back ((uint32_t)strtoul (argv[i], nullptr, 10));

  auto loaded = vkllama::load_model (argv[1], options);
  if (!loaded.ok ())
    {
      fprintf (stderr, "failed at init model: %s\n", loaded.status ().ToString ().c_str ());
      return 1;
    }
  vkllama::CausalModel &model = **loaded;
  fprintf (stderr, "all weights are uploaded to device\n");

  using clock = std::chrono::steady_clock;
  std::vector<uint32_t> toks = prompt;
  size_t offset = 0;
  const auto t0 = clock::now ();
  auto t1 = t0;
  for (int i = 0; i < predict; ++i)
    {
      auto logits = model (toks, offset);
      if (!logits.ok ())
        {
          fprintf (stderr, "failed at inferring: %s\n", logits.status ().ToString ().c_str ());
          return 1;
        }
      if (i == 0)
        t1 = clock::now ();
      // the sampler sees the last row of logits (top-1 by default; the
      // lowest index wins ties)
      const size_t V = model.vocab_size ();
      const float *row = logits->data () + (logits->size () - V);
      const uint32_t next = (uint32_t)sampler->sample (row, V);
      printf ("%u%c", next, i + 1 == predict ? '\n' : ' ');
      offset += toks.size ();
      toks = { next };
    }
  const auto t2 = clock::now ();
  fprintf (stderr, "prompt %zu tokens %.1f ms; %d tokens %.1f ms\n", prompt.size (),
           std::chrono::duration<double, std::milli> (t1 - t0).count (), predict - 1,
           std::chrono::duration<double, std::milli> (t2 - t1).count ());
  return 0;
}
